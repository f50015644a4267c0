"""Pemidra: recurrent mixers and chunked softmax attention beside a gated
delta rule, layer norms after the residual sums.

    x <- norm1(alpha * x + ls1 * mixer(x))
    x <- norm2(alpha * x + ls2 * ff(x))

* the sublayers read the residual stream itself; weighted sum, layer norm and
  the next operand are one pass (ops.ln_residual), which also folds split
  products;
* mixers: "retention" is linear attention with one decay per head
  (ops.lightning without its activation, every head normed by itself);
  "general_delta" a generalized delta rule with decay and removal rate per
  key channel (ops.general_delta); "parallel" runs softmax attention over the
  query's chunk of positions -- heads normed, half-split rotation, a sink of
  score zero, a gate per head (ops.softmax_attention) -- beside a gated delta
  rule with a short convolution and a decay per key channel
  (ops.gated_delta), norms both results and takes their mean;
* feed-forward: gelu_tanh(gate) * up (ops.gateup_swiglu).

The residual stream, norms, angles, scores, decays and states are fp32.  A
mixer's input projections, those of both sides of "parallel" together, are
one matrix product.  On the GPU in bf16 the decode path streams packed copies
of the weights (ops.pack_weight).
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import List, Optional, Tuple

import torch

from ..ops import interface as ops
from .hybrid import HybridLayer, HybridModel, RopeSpec, RopeTables


def _grouped(heads: int, kv_heads: int) -> None:
    if kv_heads < 1 or heads % kv_heads:
        raise ValueError(f"{heads} heads do not share {kv_heads} key heads "
                         "evenly")


@dataclass(frozen=True)
class ChunkedAttentionSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rope: RopeSpec
    chunk: int                # a query sees its own chunk of positions

    def __post_init__(self):
        _grouped(self.heads, self.kv_heads)
        if self.rope.dims > self.dim:
            raise ValueError(f"{self.rope.dims} rotated dimensions of "
                             f"{self.dim}")
        if self.chunk < 1:
            raise ValueError(f"chunks of {self.chunk} positions")

    @classmethod
    def from_json(cls, m: dict) -> "ChunkedAttentionSpec":
        return cls(m["heads"], m["kv_heads"], m["dim"], m["vdim"],
                   float(m["scale"]), RopeSpec.from_json(m["rot"], True),
                   int(m["mask"]["size"]))


@dataclass(frozen=True)
class GatedDeltaSpec:
    heads: int
    kv_heads: int             # of queries and keys
    dim: int
    vdim: int
    conv: int                 # taps of the short convolution

    def __post_init__(self):
        _grouped(self.heads, self.kv_heads)
        if self.conv < 1:
            raise ValueError(f"a convolution of {self.conv} taps")

    @classmethod
    def from_json(cls, m: dict) -> "GatedDeltaSpec":
        return cls(m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"])

    @property
    def channels(self) -> int:
        return 2 * self.kv_heads * self.dim + self.heads * self.vdim


@dataclass(frozen=True)
class GeneralDeltaSpec:
    heads: int
    dim: int

    @classmethod
    def from_json(cls, m: dict) -> "GeneralDeltaSpec":
        return cls(m["heads"], m["dim"])


@dataclass(frozen=True)
class RetentionSpec:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]  # per head

    def __post_init__(self):
        if len(self.decay) != self.heads:
            raise ValueError(f"{len(self.decay)} decays for {self.heads} "
                             "heads")

    @classmethod
    def from_json(cls, m: dict) -> "RetentionSpec":
        return cls(m["heads"], m["dim"], m["vdim"],
                   tuple(float(x) for x in m["decay"]))


@dataclass(frozen=True)
class ParallelSpec:
    left: ChunkedAttentionSpec
    right: GatedDeltaSpec

    @classmethod
    def from_json(cls, m: dict) -> "ParallelSpec":
        return cls(ChunkedAttentionSpec.from_json(m["left"]),
                   GatedDeltaSpec.from_json(m["right"]))

    @property
    def heads(self) -> int:
        return self.left.heads


SPECS = {"retention": RetentionSpec, "general_delta": GeneralDeltaSpec,
         "parallel": ParallelSpec}


@dataclass(frozen=True)
class PemidraLayerSpec:
    type: str                 # a key of SPECS
    mixer: object             # and its class
    ff: Optional[int] = None  # None: no feed-forward

    @classmethod
    def from_json(cls, d: dict) -> "PemidraLayerSpec":
        if d["type"] not in SPECS:
            raise ValueError(f"unknown mixer {d['type']!r}")
        mlp = d.get("mlp")
        if mlp and mlp.get("kind") != "dense":
            raise ValueError(f"unknown feed-forward {mlp.get('kind')!r}")
        return cls(d["type"], SPECS[d["type"]].from_json(d["mixer"]),
                   mlp["ff"] if mlp else None)


@dataclass
class PemidraConfig:
    name: str
    width: int
    vocab: int
    layers: List[PemidraLayerSpec]
    eps: float = 1e-6
    alpha: float = 1.0                    # of the residual in the sums
    low_rank: int = 16                    # of a random model's projections
    max_ctx: int = 131072                 # length of the rotation tables
    checkpoint: Optional[str] = None      # folder with the weights

    family = "pemidra"
    sliding_window = 0                    # chunks are per layer

    @classmethod
    def from_json(cls, d: dict, name: str = "pemidra",
                  checkpoint: Optional[str] = None) -> "PemidraConfig":
        return cls(
            name=name, width=d["width"], vocab=d["vocab"],
            layers=[PemidraLayerSpec.from_json(e) for e in d["layers"]],
            eps=d["norm"]["eps"], alpha=d["postln_alpha"],
            checkpoint=checkpoint)

    def run_stores(self):
        """What each layer keeps per sequence."""
        from ..engine.kvcache import RunStore
        out = []
        for s in self.layers:
            m = s.mixer
            if s.type == "retention":
                out.append(RunStore(state=(
                    ("retention", (m.heads, m.dim, m.vdim)),)))
            elif s.type == "general_delta":
                out.append(RunStore(state=(
                    ("delta", (m.heads, m.dim, m.dim)),)))
            else:
                a, r = m.left, m.right
                out.append(RunStore(
                    kv=(a.kv_heads, a.dim, a.vdim),
                    state=(("delta", (r.heads, r.dim, r.vdim)),
                           ("conv", (r.conv - 1, r.channels)))))
        return out

    def weight_bytes(self) -> int:
        """Size of the bf16 weights."""
        W, R = self.width, self.low_rank
        n = 2 * self.vocab * W
        for s in self.layers:
            m = s.mixer
            if s.type == "retention":
                n += W * m.heads * (2 * m.dim + 3 * m.vdim)
            elif s.type == "general_delta":
                n += m.heads * m.dim * (6 * W + R) + W * R
            else:
                a, r = m.left, m.right
                n += W * (a.heads * (a.dim + a.vdim + 1)
                          + a.kv_heads * (a.dim + a.vdim) + r.channels
                          + r.heads * (r.vdim + 1) + 2 * R)
                n += R * r.heads * (r.dim + r.vdim) + r.conv * r.channels
            n += 3 * W * (s.ff or 0)
        return 2 * n

    def model_info(self) -> dict:
        """Architecture facts for /api/show."""
        return {
            "block_count": len(self.layers),
            "embedding_length": self.width,
            "context_length": self.max_ctx,
            "feed_forward_length": max(s.ff or 0 for s in self.layers),
            "attention.head_count": max(s.mixer.heads for s in self.layers),
            "vocab_size": self.vocab,
        }


def _sized(heads, kv_heads, small, ff):
    """The three kinds of layers at the size of a real model's; `small` heads
    in the right half of a parallel layer."""
    return {
        "r": PemidraLayerSpec("retention", RetentionSpec(
            heads, 128, 128, tuple(1.0 - 2.0 ** -(5.0 + 5.0 * h / heads)
                                   for h in range(heads))), ff),
        "g": PemidraLayerSpec("general_delta",
                              GeneralDeltaSpec(2 * heads, 64), ff),
        "p": PemidraLayerSpec("parallel", ParallelSpec(
            ChunkedAttentionSpec(heads, kv_heads, 128, 128, 128 ** -0.5,
                                 RopeSpec(64, 1e6, None, True), 4096),
            GatedDeltaSpec(small, small, 128, 128, 4)), ff)}


def _stack(kinds, pattern):
    return [kinds[c] for c in pattern]


PEMIDRA_PRESETS = {
    # small enough for CPU tests
    "pemidra-tiny": PemidraConfig(
        name="pemidra-tiny", width=192, vocab=320, alpha=2.0, max_ctx=2048,
        layers=_stack({
            "r": PemidraLayerSpec("retention", RetentionSpec(
                3, 24, 40, (0.5, 0.9, 0.99))),
            "g": PemidraLayerSpec("general_delta", GeneralDeltaSpec(4, 32)),
            "p": PemidraLayerSpec("parallel", ParallelSpec(
                ChunkedAttentionSpec(4, 2, 32, 24, 0.2,
                                     RopeSpec(16, 1e4, None, True), 50),
                GatedDeltaSpec(4, 2, 16, 32, 3)), 200)}, "prgp")),
    # layers the size of an 8B and of a 1B model's
    "pemidra-8b": PemidraConfig(
        name="pemidra-8b", width=4096, vocab=128256, alpha=2.0, low_rank=128,
        layers=_stack(_sized(32, 8, 16, 11264), "prgp" * 8)),
    "pemidra-1b": PemidraConfig(
        name="pemidra-1b", width=2048, vocab=128256, alpha=2.0, low_rank=64,
        layers=_stack(_sized(16, 4, 8, 6144), "prgp" * 4)),
}


def _offsets(parts):
    """First column of every part (a matrix or its rows)."""
    out, at = [], 0
    for p in parts:
        out.append(at)
        at += p if isinstance(p, int) else p.shape[0]
    return out


def _whole(m, dim):
    """A low-rank projection with its rank filled up to whole vectors."""
    fill = -m.shape[dim] % 8
    return torch.nn.functional.pad(m, (0, fill) if dim == 1
                                   else (0, 0, 0, fill))


def _low_rank(m):
    return ops.low_rank(_whole(m, 1).contiguous())


def _aligned(cols, low):
    """Wide projections, then low-rank ones from whole vectors on."""
    fill = -sum(m.shape[0] for m in cols) % 8
    if fill:
        cols = cols + [low[0].new_zeros(fill, low[0].shape[1])]
    return cols + [_whole(m, 0) for m in low]


class PemidraLayer(HybridLayer):
    def __init__(self, spec: PemidraLayerSpec, width: int, eps: float,
                 pre: str, get, put, vec, norm, rope):
        self.spec = spec
        W, m, mix = width, spec.mixer, pre + "mix."

        def mat(name, rows, cols=W):
            return get(mix + name, (rows, cols))

        def scale(name):
            return vec(pre + name, W, mean=1.0)

        self.norm1, self.ls1 = norm(pre + "norm1"), scale("ls1")
        if spec.type == "retention":
            qk, v = m.heads * m.dim, m.heads * m.vdim
            cols = [mat("q", qk), mat("k", qk), mat("v", v), mat("g", v)]
            self.mix = ops.LightningWeights(
                heads=m.heads, dim=m.dim, vdim=m.vdim,
                offsets=tuple(_offsets(cols)),
                powers=ops.decay_powers(m.decay, self.ls1.device), norm=None,
                eps=eps, act=False, scale=m.dim ** -0.5, per_head=True,
                gate="silu")
            outs = [("w_o", "o", v)]
        elif spec.type == "general_delta":
            n = m.heads * m.dim
            low = mat("w1", None)
            cols = _aligned([mat(c, n) for c in "rkvag"], [low])
            self.mix = ops.GeneralDeltaWeights(
                heads=m.heads, dim=m.dim,
                offsets=(*_offsets(cols)[:5], _offsets(cols)[-1]),
                w2=_low_rank(put(mat("w2", n, low.shape[0]))),
                w0=vec(mix + "w0", n), a_bias=vec(mix + "a.b", n),
                norm=vec(mix + "norm", n, mean=1.0), eps=eps)
            outs = [("w_o", "o", n)]
        else:
            cols, outs = self._parallel(m, mat, mix, vec, put, rope, eps)
        self.w_in = self.fused_rows(cols, put)
        self.outs = [name for name, _, _ in outs]
        for name, stored, k in outs:
            setattr(self, name, put(mat(stored, W, k)).contiguous())
        if spec.ff:
            self.norm2, self.ls2 = norm(pre + "norm2"), scale("ls2")
            # zero columns fill the feed-forward up to whole tiles
            F, mlp = -(-spec.ff // 64) * 64, pre + "mlp."
            gate, up = (put(get(mlp + n, (spec.ff, W)))
                        for n in ("gate", "up"))
            down = put(get(mlp + "down", (W, spec.ff)))
            self.w_gu = gate.new_zeros(2 * F, W)
            self.w_gu[:spec.ff], self.w_gu[F:F + spec.ff] = gate, up
            self.w_down = down.new_zeros(W, F)
            self.w_down[:, :spec.ff] = down

    def _parallel(self, m, mat, mix, vec, put, rope, eps):
        a, r = m.left, m.right
        cols = [mat(n, rows) for n, rows in (
            ("left.q", a.heads * a.dim), ("left.k", a.kv_heads * a.dim),
            ("left.v", a.kv_heads * a.vdim), ("right.q", r.kv_heads * r.dim),
            ("right.k", r.kv_heads * r.dim), ("right.v", r.heads * r.vdim),
            ("left.g", a.heads), ("right.b", r.heads))]
        a1, g1 = mat("right.a1", None), mat("right.g1", None)
        at = _offsets(cols)
        cols = _aligned(cols, [a1, g1])
        at_a1, at_g1 = _offsets(cols)[-2:]
        self.gate_at = at[6]
        self.rope = rope(a.rope)
        temp = vec(mix + "left.temp", a.heads, mean=1.0)
        self.heads = ops.HeadNorms(
            q=vec(mix + "left.q.norm", a.dim, mean=1.0),
            k=vec(mix + "left.k.norm", a.dim, mean=1.0),
            values=True, gain=temp, eps=eps)
        self.attn = ops.SoftmaxAttn(
            heads=a.heads, kv_heads=a.kv_heads, dim=a.dim, vdim=a.vdim,
            scale=a.scale, sink=torch.zeros_like(temp), chunk=a.chunk)
        taps = torch.cat([mat(f"right.{n}.conv", rows, r.conv) for n, rows in
                          (("q", r.kv_heads * r.dim),
                           ("k", r.kv_heads * r.dim),
                           ("v", r.heads * r.vdim))])
        self.delta = ops.GatedDeltaWeights(
            heads=r.heads, kv_heads=r.kv_heads, dim=r.dim, vdim=r.vdim,
            offsets=(at[3], at[7], at_a1, at_g1),
            conv=taps.to(temp.device).float().t().contiguous(),
            a2=_low_rank(put(mat("right.a2", r.heads * r.dim,
                                 a1.shape[0]))),
            rate=vec(mix + "right.A_log", r.heads).exp(),
            dt_bias=vec(mix + "right.dt_bias", r.heads * r.dim),
            g2=_low_rank(put(mat("right.g2", r.heads * r.vdim,
                                 g1.shape[0]))),
            norm=vec(mix + "right.norm", r.vdim, mean=1.0), eps=eps)
        W = cols[0].shape[1]
        self.left_out, self.right_out = (vec(f"{mix}{n}.out", W, mean=1.0)
                                         for n in ("left", "right"))
        return cols, [("w_lo", "left.o", a.heads * a.vdim),
                      ("w_ro", "right.o", r.heads * r.vdim)]

    def matrices(self):
        names = ["w_in"] + self.outs \
            + (["w_gu", "w_down"] if self.spec.ff else [])
        return {n: getattr(self, n) for n in names}

    def pack(self, name, w):
        return ops.pack_weight_gu(w) if name == "w_gu" \
            else super().pack(name, w)


class PemidraModel(HybridModel):
    def __init__(self, cfg: PemidraConfig, device: str = "cpu",
                 dtype: torch.dtype = torch.float32, seed: int = 1234,
                 tp_rank: int = 0, tp_size: int = 1, process_group=None,
                 fast_init: bool = False):
        super().__init__(cfg, device, dtype, tp_size, process_group)
        get = self._source(seed, fast_init, cfg.low_rank)
        put, W = self._put, cfg.width

        def vec(name, n, mean=0.0):
            return get(name, (n,), mean=mean, spread=0.1) \
                .to(self.device).float().contiguous()

        def norm(name):
            return ops.LayerNorm(vec(name, W, mean=1.0), vec(name + ".b", W))

        rope = RopeTables(cfg.max_ctx, self.device)
        self.embed = put(get("embed", (cfg.vocab, W),
                             spread=1.0)).contiguous()
        self.layers = [
            PemidraLayer(s, W, cfg.eps, f"l{i}.", get, put, vec, norm, rope)
            for i, s in enumerate(cfg.layers)]
        self.final_norm = norm("final.norm")
        self.head = put(get("head", (cfg.vocab, W))).contiguous()
        self._pack_weights()

    def _mixer(self, layer, run, h, cache, slot_ids, positions, meta, frag):
        p = ops.linear_parts(h, layer.w_in, layer.packs.get("w_in"), most=3)
        state = cache.state[run]

        def out(name, o):
            return ops.linear_parts(o, getattr(layer, name),
                                    layer.packs.get(name))

        if layer.spec.type == "retention":
            return out("w_o", ops.lightning(
                p, layer.mix, state["retention"], slot_ids, positions, meta,
                frag))
        if layer.spec.type == "general_delta":
            return out("w_o", ops.general_delta(
                p, layer.mix, state["delta"], slot_ids, positions, meta,
                frag))
        q = ops.qkv_norm_rope_append(p, layer.heads, cache, run, layer.attn,
                                     layer.rope, slot_ids, positions)
        left = ops.softmax_attention(q, cache, run, layer.attn, slot_ids,
                                     positions, meta, frag,
                                     gate=ops.Columns(p, layer.gate_at))
        right = ops.gated_delta(p, layer.delta, state["delta"],
                                state["conv"], slot_ids, positions, meta,
                                frag)
        return ops.Branches(((out("w_lo", left), layer.left_out),
                             (out("w_ro", right), layer.right_out)), 0.5)

    def forward(
        self,
        tokens: torch.Tensor,      # [T] flat token ids
        positions: torch.Tensor,   # [T] position of each token in its seq
        kv_cache,                  # engine.kvcache.HybridCache
        slot_ids: torch.Tensor,    # [T] slot of each token's sequence
        attn_meta,                 # ops.AttnMeta
        return_hidden: bool = False,
        layer_out: Optional[list] = None,
    ) -> torch.Tensor:
        """Logits (or final-norm hidden states) of the rows attn_meta
        selects.  layer_out collects the residual stream after every
        layer."""
        meta = attn_meta
        frag = (self.frag_decode and meta.one_each
                and tokens.shape[0] <= 64)

        def join(x, y=None, norm=None, scale=None, **kw):
            return ops.ln_residual(x, y, norm, self.cfg.alpha, self.cfg.eps,
                                   scale, embed=self.embed, tokens=tokens,
                                   **{"frag": frag, **kw})

        x, todo = None, ()         # todo: the sum that is still to be made
        for run, layer in enumerate(self.layers):
            x, h = join(x, *todo)
            y = self._mixer(layer, run, h, kv_cache, slot_ids, positions,
                            meta, frag)
            todo = (y, layer.norm1, layer.ls1)
            if layer.spec.ff:
                x, h = join(x, *todo)
                a = ops.gateup_swiglu(h, layer.w_gu, layer.packs.get("w_gu"),
                                      act="gelu_tanh")
                y = ops.linear_parts(a, layer.w_down,
                                     layer.packs.get("w_down"))
                todo = (y, layer.norm2, layer.ls2)
            if layer_out is not None:
                layer_out.append(join(x, *todo, frag=False)[0])
        frag = frag and not return_hidden and self.head_pk is not None
        _, h = join(x, *todo, then=self.final_norm, rows=meta.logits_idx,
                    need_x=False, frag=frag)
        if return_hidden:
            return h
        return ops.linear(h, self.head,
                          packed=self.head_pk if frag else None)
