"""Kavedra: lightning attention, softmax attention with a sink and windowed
latent attention in one stack, with an optional loop over some layers.

    x <- x + mixer(norm1(x))
    x <- x + ff(norm2(x))

* norms are RMS norms whose stored weight is the distance from one; norm,
  residual sum and the fold of split products are one pass
  (ops.rms_residual);
* mixers: "lightning" keeps an fp32 [heads, dim, vdim] state per sequence
  with one decay per head (ops.lightning); "attention" is softmax attention
  over paged keys and values with biases, interleaved rotary positions and a
  learned sink (ops.softmax_attention); "latent_attention" pages one latent
  row and one rotated key part per token, sees a window and gates its output
  (ops.latent_attention);
* feed-forward: silu(gate) * up (ops.gateup_swiglu);
* layers start..stop-1 may run several times with the same weights.  Before
  every pass the residual stream is replaced by a linear map of itself and
  the embedding output, plus a vector of the pass.  Every run of a layer has
  its own cache or state.

The residual stream, norms, angles, scores, gates and states are fp32.  A
mixer's input projections are one matrix product.  On the GPU in bf16 the
decode path streams packed copies of the weights (ops.pack_weight).
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import List, Optional, Tuple

import torch

from ..ops import interface as ops
from .hybrid import HybridLayer, HybridModel, RopeSpec, RopeTables


@dataclass(frozen=True)
class KavedraLayerSpec:
    type: str                 # lightning, attention, latent_attention
    heads: int
    dim: int                  # latent_attention: the unrotated part
    vdim: int
    decay: Tuple[float, ...] = ()         # lightning, per head
    kv_heads: int = 0                     # attention
    scale: float = 1.0                    # attention, latent_attention
    rope: Optional[RopeSpec] = None
    kv_rank: int = 0                      # latent_attention
    rot_dim: int = 0
    window: int = 0           # tokens a query sees, itself included; 0: all
    ff: Optional[int] = None  # None: no feed-forward

    def __post_init__(self):
        if self.type == "lightning":
            if len(self.decay) != self.heads:
                raise ValueError(f"{len(self.decay)} decays for "
                                 f"{self.heads} heads")
        elif self.type == "attention":
            if self.kv_heads < 1 or self.heads % self.kv_heads:
                raise ValueError(f"{self.heads} heads do not share "
                                 f"{self.kv_heads} key/value heads evenly")
            if self.rope.dims > self.dim:
                raise ValueError(f"{self.rope.dims} rotated dimensions of "
                                 f"{self.dim}")
        elif self.type == "latent_attention":
            if self.rope.dims != self.rot_dim:
                raise ValueError(f"{self.rope.dims} rotated dimensions, "
                                 f"rot_dim {self.rot_dim}")
        else:
            raise ValueError(f"unknown mixer {self.type!r}")
        if self.window < 0:
            raise ValueError(f"window of {self.window} tokens")

    @classmethod
    def from_json(cls, d: dict) -> "KavedraLayerSpec":
        m, mlp = d["mixer"], d.get("mlp")
        if mlp and mlp.get("kind") != "dense":
            raise ValueError(f"unknown feed-forward {mlp.get('kind')!r}")
        kw = {k: m[k] for k in ("heads", "dim", "vdim", "kv_heads", "kv_rank",
                                "rot_dim") if k in m}
        if "decay" in m:
            kw["decay"] = tuple(float(x) for x in m["decay"])
        if "scale" in m:
            kw["scale"] = float(m["scale"])
        if "rot" in m:
            kw["rope"] = RopeSpec.from_json(m["rot"])
        if m.get("mask"):
            kw["window"] = int(m["mask"]["size"])
            if kw["window"] < 1:
                raise ValueError(f"window of {kw['window']} tokens")
        return cls(type=d["type"], ff=mlp["ff"] if mlp else None, **kw)

    @property
    def row(self) -> int:
        """Cached row of latent attention, in whole 16-byte vectors."""
        return -(-(self.kv_rank + self.rot_dim) // 8) * 8


@dataclass
class KavedraConfig:
    name: str
    width: int
    vocab: int
    layers: List[KavedraLayerSpec]
    eps: float = 1e-6
    logit_scale: float = 1.0
    loop: Optional[Tuple[int, int, int]] = None   # start, stop, times
    max_ctx: int = 131072                 # length of the rotation tables
    checkpoint: Optional[str] = None      # folder with the weights

    family = "kavedra"
    sliding_window = 0                    # windows are per layer

    def __post_init__(self):
        if self.loop is not None:
            start, stop, times = self.loop
            if not (0 <= start <= stop <= len(self.layers)) or times < 0:
                raise ValueError(f"loop {self.loop} does not fit "
                                 f"{len(self.layers)} layers")

    @classmethod
    def from_json(cls, d: dict, name: str = "kavedra",
                  checkpoint: Optional[str] = None) -> "KavedraConfig":
        lp = d.get("loop")
        return cls(
            name=name, width=d["width"], vocab=d["vocab"],
            layers=[KavedraLayerSpec.from_json(e) for e in d["layers"]],
            eps=d["norm"]["eps"], logit_scale=d["logit_scale"],
            loop=(lp["start"], lp["stop"], lp["times"]) if lp else None,
            checkpoint=checkpoint)

    @property
    def runs(self) -> List[Tuple[int, Optional[int]]]:
        """(layer, pass it opens or None) of every layer run, in order."""
        n = len(self.layers)
        if self.loop is None:
            return [(i, None) for i in range(n)]
        start, stop, times = self.loop
        return ([(i, None) for i in range(start)]
                + [(i, t if i == start else None) for t in range(times)
                   for i in range(start, stop)]
                + [(i, None) for i in range(stop, n)])

    def run_stores(self):
        """What each layer run keeps per sequence."""
        from ..engine.kvcache import RunStore
        out = []
        for li, _ in self.runs:
            s = self.layers[li]
            if s.type == "lightning":
                out.append(RunStore(state=(
                    ("lightning", (s.heads, s.dim, s.vdim)),)))
            elif s.type == "attention":
                out.append(RunStore(kv=(s.kv_heads, s.dim, s.vdim)))
            else:
                out.append(RunStore(latent=s.row))
        return out

    def weight_bytes(self) -> int:
        """Size of the bf16 weights."""
        W, n = self.width, 2 * self.vocab * self.width
        if self.loop is not None:
            n += 2 * W * W
        for s in self.layers:
            qk, v = s.heads * s.dim, s.heads * s.vdim
            if s.type == "lightning":
                n += W * (2 * qk + 3 * v)
            elif s.type == "attention":
                n += W * (qk + v + s.kv_heads * (s.dim + s.vdim))
            else:
                n += W * (qk + s.heads * s.rot_dim + s.kv_rank + s.rot_dim
                          + 2 * v) + s.kv_rank * (qk + v)
            n += 3 * W * (s.ff or 0)
        return 2 * n

    def model_info(self) -> dict:
        """Architecture facts for /api/show."""
        return {
            "block_count": len(self.layers),
            "block_runs": len(self.runs),
            "embedding_length": self.width,
            "context_length": self.max_ctx,
            "feed_forward_length": max(s.ff or 0 for s in self.layers),
            "attention.head_count": max(s.heads for s in self.layers),
            "vocab_size": self.vocab,
        }


def _decays(heads: int) -> Tuple[float, ...]:
    """Memories from a few tokens to some thousands, evenly in octaves."""
    return tuple(1.0 - 2.0 ** -(2.0 + 9.0 * h / max(1, heads - 1))
                 for h in range(heads))


def _stack(width, vocab, kinds, pattern, **kw):
    return dict(width=width, vocab=vocab,
                layers=[kinds[c] for c in pattern], **kw)


def _sized(heads, kv_heads, ff):
    """The three kinds of layers at the size of a real model's."""
    return {
        "s": KavedraLayerSpec("lightning", heads, 128, 128,
                              decay=_decays(heads), ff=ff),
        "a": KavedraLayerSpec("attention", heads, 128, 128,
                              kv_heads=kv_heads, scale=128 ** -0.5,
                              rope=RopeSpec(128, 1e6), ff=ff),
        "l": KavedraLayerSpec("latent_attention", heads, 128, 128,
                              kv_rank=512, rot_dim=64, scale=192 ** -0.5,
                              rope=RopeSpec(64, 1e4, (40.0, 4096, 32.0, 1.0)),
                              window=4096, ff=ff)}


KAVEDRA_PRESETS = {
    # small enough for CPU tests
    "kavedra-tiny": KavedraConfig(name="kavedra-tiny", **_stack(
        192, 320,
        {"s": KavedraLayerSpec("lightning", 3, 24, 40,
                               decay=(0.5, 0.9, 0.99), ff=200),
         "a": KavedraLayerSpec("attention", 4, 32, 24, kv_heads=2, scale=0.2,
                               rope=RopeSpec(16, 1e4), ff=200),
         "l": KavedraLayerSpec("latent_attention", 3, 24, 32, kv_rank=40,
                               rot_dim=16, scale=0.17, window=50, ff=200,
                               rope=RopeSpec(16, 1e4,
                                             (4.0, 512, 16.0, 1.0)))},
        "slsa", loop=(1, 3, 2), logit_scale=0.5, max_ctx=2048)),
    # layers the size of an 8B and of a 1B model's, one pass, two recurrent
    # layers for every attention of each kind
    "kavedra-8b": KavedraConfig(name="kavedra-8b", **_stack(
        4096, 128256, _sized(32, 8, 14336), "slsa" * 8)),
    "kavedra-1b": KavedraConfig(name="kavedra-1b", **_stack(
        2048, 128256, _sized(16, 4, 8192), "slsa" * 4)),
}


class KavedraLayer(HybridLayer):
    def __init__(self, spec: KavedraLayerSpec, width: int, eps: float,
                 pre: str, get, put, vec, gain, rope):
        self.spec = spec
        s, W = spec, width
        qk, v = s.heads * s.dim, s.heads * s.vdim
        mix = pre + "mix."

        def mat(name, rows, cols=W):
            return get(mix + name, (rows, cols))

        self.norm1 = gain(pre + "norm1")
        if s.type == "lightning":
            cols = [mat("q", qk), mat("k", qk), mat("v", v), mat("g", v)]
            norm = vec(mix + "norm", v, mean=1.0)
            self.mix = ops.LightningWeights(
                heads=s.heads, dim=s.dim, vdim=s.vdim,
                offsets=(0, qk, 2 * qk, 2 * qk + v),
                powers=ops.decay_powers(s.decay, norm.device), norm=norm,
                eps=eps)
        elif s.type == "attention":
            nk, nv = s.kv_heads * s.dim, s.kv_heads * s.vdim
            parts = (("q", qk), ("k", nk), ("v", nv))
            cols = [mat(n, rows) for n, rows in parts]
            self.bias = torch.cat([vec(f"{mix}{n}.b", rows)
                                   for n, rows in parts])
            self.rope = rope(s.rope)
            self.mix = ops.SoftmaxAttn(
                heads=s.heads, kv_heads=s.kv_heads, dim=s.dim, vdim=s.vdim,
                scale=s.scale, sink=vec(mix + "sink", s.heads),
                window=s.window)
        else:
            R, E = s.kv_rank, s.rot_dim
            nq = qk + s.heads * E
            cols = [mat("q", nq), mat("dkv", R + E), mat("g", v)]
            self.gate_at = nq + R + E
            self.dkv_norm = vec(mix + "dkv.norm", R, mean=1.0)
            self.rope = rope(s.rope)
            uk = put(mat("uk", qk, R)).view(s.heads, s.dim, R)
            uv = put(mat("uv", v, R)).view(s.heads, s.vdim, R)
            self.mix = ops.LatentWeights(
                uk=uk.contiguous(), uk_t=uk.transpose(1, 2).contiguous(),
                uv=uv.contiguous(), scale=s.scale, rot_dim=E,
                window=s.window)
        self.w_in = self.fused_rows(cols, put)
        self.w_o = put(mat("o", W, v)).contiguous()
        if s.ff:
            self.norm2 = gain(pre + "norm2")
            # zero columns fill the feed-forward up to whole tiles
            F, mlp = -(-s.ff // 64) * 64, pre + "mlp."
            gate, up = (put(get(mlp + n, (s.ff, W))) for n in ("gate", "up"))
            down = put(get(mlp + "down", (W, s.ff)))
            self.w_gu = gate.new_zeros(2 * F, W)
            self.w_gu[:s.ff], self.w_gu[F:F + s.ff] = gate, up
            self.w_down = down.new_zeros(W, F)
            self.w_down[:, :s.ff] = down

    def matrices(self):
        names = ["w_in", "w_o"] + (["w_gu", "w_down"] if self.spec.ff else [])
        return {n: getattr(self, n) for n in names}

    def pack(self, name, w):
        return ops.pack_weight_gu(w) if name == "w_gu" \
            else super().pack(name, w)


class KavedraModel(HybridModel):
    def __init__(self, cfg: KavedraConfig, device: str = "cpu",
                 dtype: torch.dtype = torch.float32, seed: int = 1234,
                 tp_rank: int = 0, tp_size: int = 1, process_group=None,
                 fast_init: bool = False):
        super().__init__(cfg, device, dtype, tp_size, process_group)
        get, put = self._source(seed, fast_init), self._put
        W = cfg.width

        def vec(name, n, mean=0.0):
            return get(name, (n,), mean=mean, spread=0.1) \
                .to(self.device).float().contiguous()

        def gain(name):
            return 1.0 + vec(name, W)

        rope = RopeTables(cfg.max_ctx, self.device)
        self.embed = put(get("embed", (cfg.vocab, W),
                             spread=1.0)).contiguous()
        self.loop_in = self.loop_step = None
        if cfg.loop is not None:
            self.loop_in = put(get("loop.in", (W, 2 * W))).contiguous()
            self.loop_step = get("loop.step", (cfg.loop[2], W), spread=0.1) \
                .to(self.device).float().contiguous()
        self.layers = [
            KavedraLayer(s, W, cfg.eps, f"l{i}.", get, put, vec, gain, rope)
            for i, s in enumerate(cfg.layers)]
        self.final_norm = gain("final.norm")
        # the scale of the logits goes with the last norm's gain
        self.head_norm = self.final_norm * cfg.logit_scale
        self.head = put(get("head", (cfg.vocab, W))).contiguous()
        self._pack_weights()

    def matrices(self):
        return {} if self.loop_in is None else {"loop_in": self.loop_in}

    def _mixer(self, layer, run, h, cache, slot_ids, positions, meta, frag):
        p = ops.linear_parts(h, layer.w_in, layer.packs.get("w_in"))
        s, w = layer.spec, layer.mix
        if s.type == "lightning":
            o = ops.lightning(p, w, cache.state[run]["lightning"], slot_ids,
                              positions, meta, frag)
        elif s.type == "attention":
            q = ops.rope_qkv_append(p, layer.bias, cache, run, w, layer.rope,
                                    slot_ids, positions)
            o = ops.softmax_attention(q, cache, run, w, slot_ids, positions,
                                      meta, frag)
        else:
            q = ops.latent_rope_append(p, cache, run, w, layer.dkv_norm,
                                       self.cfg.eps, layer.rope, slot_ids,
                                       positions)
            o = ops.latent_attention(q, cache, run, w, slot_ids, positions,
                                     meta, frag,
                                     gate=ops.Columns(p, layer.gate_at))
        return ops.linear_parts(o, layer.w_o, layer.packs.get("w_o"))

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
        selects.  layer_out collects the residual stream after every layer
        run."""
        meta = attn_meta
        frag = (self.frag_decode and meta.one_each
                and tokens.shape[0] <= 64)

        def join(x, y, pre, **kw):
            return ops.rms_residual(x, y, None, pre, 1.0, self.cfg.eps,
                                    embed=self.embed, tokens=tokens,
                                    **{"frag": frag, **kw})

        x = y = None
        for run, (li, opens) in enumerate(self.cfg.runs):
            layer = self.layers[li]
            if opens is None:
                x, h = join(x, y, layer.norm1)
            else:
                _, both = join(x, y, None, tail=True, need_x=False)
                z = ops.linear_f32(both, self.loop_in,
                                   self.packs.get("loop_in"))
                x, h = join(None, z, layer.norm1, bare=True,
                            shift=self.loop_step[opens])
            y = self._mixer(layer, run, h, kv_cache, slot_ids, positions,
                            meta, frag)
            if layer.spec.ff:
                x, h = join(x, y, layer.norm2)
                a = ops.gateup_swiglu(h, layer.w_gu, layer.packs.get("w_gu"))
                y = ops.linear_parts(a, layer.w_down,
                                     layer.packs.get("w_down"))
            if layer_out is not None:
                layer_out.append(join(x, y, None, frag=False)[0])
        frag = frag and not return_hidden and self.head_pk is not None
        _, h = join(x, y, self.final_norm if return_hidden
                    else self.head_norm, rows=meta.logits_idx, need_x=False,
                    frag=frag)
        if return_hidden:
            return h
        return ops.linear(h, self.head,
                          packed=self.head_pk if frag else None)
