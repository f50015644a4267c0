"""The Pemidra design against a plain float64 statement of its equations
(pemidra_oracle.py): every mechanism alone, then whole models fed in
portions, in batches and through reused memory, then generation.

The same tests run on the CPU and, in fp32 and bf16, on the GPU kernels.
"""
import json
import math
import os
import subprocess

import pytest
import torch
from safetensors.torch import save_file

import pemidra_oracle as oracle
from hybrid_common import (BF16, F32, F64, GPU, cut, exact, generate,
                           meta_for, rel, rows_of, run_portions, tol, where)
from ollamamq_amd.engine import (GenParams, HybridCache, LlamaEngine,
                                 cache_for_model)
from ollamamq_amd.engine.kvcache import RunStore
from ollamamq_amd.engine.trace import make_engine
from ollamamq_amd.models import (PemidraConfig, build_model,
                                 config_from_folder)
from ollamamq_amd.models.hybrid import RopeSpec, RopeTables
from ollamamq_amd.ops import interface as ops

REPO = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def layer(kind, mixer, ff):
    return {"type": kind, "mixer": mixer,
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def reten(heads, dim, vdim, decay, ff=None):
    return layer("retention", dict(heads=heads, dim=dim, vdim=vdim,
                                   decay=decay), ff)


def general(heads, dim, ff=None):
    return layer("general_delta", dict(heads=heads, dim=dim), ff)


def both(left, right, ff=None):
    """left: heads, kv_heads, dim, vdim, (rotated, base), chunk, scale;
    right: heads, kv_heads, dim, vdim, taps"""
    H, G, D, V, rot, chunk, scale = left
    return layer("parallel", {
        "left": dict(heads=H, kv_heads=G, dim=D, vdim=V, scale=scale,
                     rot=dict(dims=rot[0], base=rot[1]),
                     mask={"size": chunk}),
        "right": dict(zip(("heads", "kv_heads", "dim", "vdim", "conv"),
                          right))}, ff)


def config(width, vocab, layers, eps=1e-5, alpha=2.0):
    return {"architecture": "Pemidra", "width": width, "vocab": vocab,
            "layers": layers, "norm": {"eps": eps}, "postln_alpha": alpha}


MODELS = {
    # no two layers alike, feed-forwards behind some of each kind
    "mixed": config(128, 200, [
        reten(3, 24, 40, [0.3, 0.9, 0.995], 80),
        both((6, 2, 24, 40, (8, 500.0), 37, 0.3), (4, 2, 16, 24, 3)),
        general(5, 16, 96),
        both((4, 4, 40, 16, (40, 1e4), 16, 0.2), (3, 1, 40, 8, 5), 72),
        general(2, 40)], alpha=1.7),
    # sizes that fit no tile, chunks of one token and of all, one tap,
    # nothing rotated
    "odd": config(90, 131, [
        both((3, 1, 9, 7, (4, 100.0), 1, 0.5), (3, 3, 7, 5, 1), 34),
        reten(3, 9, 7, [0.0, 1.0, 0.8]),
        both((2, 2, 22, 14, (0, 1.0), 1000, 0.4), (2, 1, 5, 10, 2)),
        general(3, 10, 50)], eps=1e-3, alpha=1.5),
    # groups of heads that need more than one tile, wide states, ranks of
    # more than one pass
    "wide": config(192, 96, [
        both((20, 1, 64, 136, (64, 1e6), 100, 0.1), (3, 1, 200, 72, 4), 64),
        general(2, 136),
        reten(2, 200, 72, [0.999, 0.6], 64)], alpha=1.0),
    # every matrix fits the packed form of the decode path
    "packed": config(128, 96, [
        both((8, 4, 32, 24, (16, 1e4), 33, 0.25), (4, 2, 32, 48, 4), 160),
        reten(4, 32, 48, [0.99, 0.9, 0.7, 0.2]),
        general(4, 32, 128)], alpha=3.0),
}
RANKS = {"wide": (136, 160, 200), "packed": (24, 16, 8)}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    out = {}
    for name, cfg in MODELS.items():
        d = tmp_path_factory.mktemp(name)
        w = oracle.random_weights(cfg, len(name), RANKS.get(name, (6, 13, 9)))
        (d / "config.json").write_text(json.dumps(cfg))
        save_file({k: t.contiguous() for k, t in w.items()},
                  str(d / "model.safetensors"))
        out[name] = (str(d), cfg, w)
    return out


_ORACLE = {}


def expected(models, name, tokens):
    """Sequences share their oracle run with those they begin."""
    for (other, toks), lg in _ORACLE.items():
        if other == name and list(toks[:len(tokens)]) == list(tokens):
            return lg[:len(tokens)]
    _, cfg, w = models[name]
    _ORACLE[name, tuple(tokens)] = oracle.run(cfg, w, tokens)[0]
    return _ORACLE[name, tuple(tokens)]


def tokens_for(name, n, seed=0):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, MODELS[name]["vocab"], (300,),
                         generator=g).tolist()[:n]


def check(got, want, dtype):
    assert rel(got, want) < tol(dtype, 3e-5, 0.03)


f64 = lambda t: t.to("cpu", F64)


# ----------------------------------------------------------------- row steps

def forms_of(rows, dt, dev, g):
    """A result as rows and, in bf16, as partial sums."""
    yield rows.to(dev, dt).contiguous(), f64(rows.to(dt))
    if dt == BF16 and dev != "cpu":
        for n in (2, 3, 7):
            parts = torch.randn(n, *rows.shape, generator=g)
            parts[0] += rows
            yield ops.Partials(parts.to(dev)), f64(parts).sum(0)


@where
@pytest.mark.parametrize("W", [64, 90, 1000, 2100, 9000])
def test_norm_after_the_sum(where, W):
    """Rows from far below the eps to large, a mean far from zero, the scale
    of the result, selected rows, a second norm."""
    dev, dt = where
    g = torch.Generator().manual_seed(W)
    eps, n = 1e-3, 9
    emb = torch.randn(11, W, generator=g).to(dt)
    vecs = [m + 0.3 * torch.randn(W, generator=g)
            for m in (1.0, 0.0, 1.0, 0.0, 1.0)]
    w, b, w2, b2, scale = vecs
    size = torch.logspace(-3, 1, n)[:, None]
    x = torch.randn(n, W, generator=g) * size + 10 * size.flip(0)
    y = torch.randn(n, W, generator=g) * size.flip(0)
    toks = torch.tensor([3, 10, 0, 3, 1, 2, 4, 9, 9], dtype=torch.int32)
    d = lambda t: t.to(dev)
    kw = dict(embed=d(emb), tokens=d(toks))
    one, two = ops.LayerNorm(d(w), d(b)), ops.LayerNorm(d(w2), d(b2))
    ln = lambda t, p, q: oracle.layer_norm(t, f64(p), f64(q), eps)
    lim = tol(dt, 1e-5, 4e-3)
    for yd, ye in forms_of(y, dt, dev, g):
        for s in (None, scale):
            s64 = 1.0 if s is None else f64(s)
            want = ln(1.7 * f64(x) + s64 * ye, w, b)
            xo, h = ops.ln_residual(d(x), yd, one, 1.7, eps,
                                    None if s is None else d(s), **kw)
            assert rel(xo, want) < 1e-5 and rel(h, want) < lim
        xo, h = ops.ln_residual(d(x), yd, one, 1.7, eps, d(scale), then=two,
                                **kw)
        assert rel(xo, want) < 1e-5 and rel(h, ln(want, w2, b2)) < lim
        rows = torch.tensor([8, 2, 2, 5])
        _, h = ops.ln_residual(d(x), yd, one, 1.7, eps, d(scale), then=two,
                               rows=d(rows), need_x=False, **kw)
        assert rel(h, ln(want, w2, b2)[rows]) < lim
        e64 = f64(emb)[toks.long()]
        xo, _ = ops.ln_residual(None, yd, one, 0.3, eps, **kw)
        assert rel(xo, ln(0.3 * e64 + ye, w, b)) < 1e-5
    xo, h = ops.ln_residual(None, None, None, 1.0, eps, **kw)
    assert torch.equal(xo.cpu(), emb[toks.long()].float())
    assert torch.equal(h.cpu(), emb[toks.long()])
    _, h = ops.ln_residual(None, None, None, 1.0, eps, then=two, **kw)
    assert rel(h, ln(e64, w2, b2)) < lim


@where
@pytest.mark.parametrize("W", [64, 90, 2100])
def test_branches(where, W):
    """Each result is normed by itself, whatever their sizes, and weighted
    with its own weight; whole results beside partial sums."""
    dev, dt = where
    g = torch.Generator().manual_seed(W)
    eps, n = 1e-4, 5
    emb = torch.randn(3, W, generator=g).to(dt)
    w, b, pa, pb, scale = (torch.randn(W, generator=g) for _ in range(5))
    x = torch.randn(n, W, generator=g)
    size = torch.logspace(-3, 2, n)[:, None]
    ra = torch.randn(n, W, generator=g) * size
    rb = torch.randn(n, W, generator=g) * size.flip(0) + 1.0
    d = lambda t: t.to(dev)
    one = ops.LayerNorm(d(w), d(b))
    for ya, ea in forms_of(ra, dt, dev, g):
        for yb, eb in forms_of(rb, dt, dev, g):
            mean = 0.5 * (oracle.rms(ea, eps) * f64(pa)
                          + oracle.rms(eb, eps) * f64(pb))
            want = oracle.layer_norm(2.5 * f64(x) + f64(scale) * mean,
                                     f64(w), f64(b), eps)
            xo, _ = ops.ln_residual(
                d(x), ops.Branches(((ya, d(pa)), (yb, d(pb))), 0.5), one, 2.5,
                eps, d(scale), embed=d(emb))
            assert rel(xo, want) < 3e-6


@where
@pytest.mark.parametrize("F,rows", [(64, 1), (192, 33), (200, 5), (1024, 70)])
def test_gelu_feed_forward(where, F, rows):
    dev, dt = where
    g = torch.Generator().manual_seed(F)
    K = 128
    w = (torch.randn(2 * F, K, generator=g) / 6).to(BF16)
    w[0] *= 20                                   # far out on both sides
    x = torch.randn(rows, K, generator=g).to(BF16)
    z = f64(x) @ f64(w).T
    want = oracle.gelu_tanh(z[:, :F]) * z[:, F:]
    plain = oracle.silu(z[:, :F]) * z[:, F:]
    assert rel(plain, want) > 0.02, "the activation must show"
    wd = w.to(dev, dt)
    got = ops.gateup_swiglu(x.to(dev, dt), wd, act="gelu_tanh")
    assert rel(got, want) < tol(dt, 3e-6, 8e-3)
    assert rel(ops.gateup_swiglu(x.to(dev, dt), wd), plain) \
        < tol(dt, 3e-6, 8e-3)
    packed = ops.pack_weight_gu(wd)
    if packed is not None and F % 64 == 0 and rows <= 64:
        _, h = ops.ln_residual(x.float().to(dev), None, None, 1.0, 0.0,
                               embed=x.to(dev), frag=True)
        act = ops.gateup_swiglu(h, wd, packed, act="gelu_tanh")
        eye = torch.eye(F, dtype=BF16, device=dev)
        got = ops.linear(act, eye, packed=ops.pack_weight(eye))
        assert rel(got, want) < 8e-3


# --------------------------------------------------- norms, rotation, append

QKV = [((6, 2, 24, 40), 8), ((3, 1, 9, 7), 4), ((4, 4, 64, 136), 64),
       ((2, 1, 32, 16), 0), ((40, 8, 128, 128), 64), ((2, 1, 256, 250), 22)]


@where
@pytest.mark.parametrize("size,dims", QKV, ids=str)
@pytest.mark.parametrize("n", [1, 70])
def test_split_norm_rotate_append(where, size, dims, n):
    """Every head by itself, small heads beside large ones; halves of the
    first dimensions turn; a factor per query head, zero and negative too;
    nothing else in the pools changes."""
    dev, dt = where
    H, G, D, V = size
    g = torch.Generator().manual_seed(n)
    w = ops.SoftmaxAttn(H, G, D, V, 1.0)
    c, eps = H * D + G * (D + V), 1e-2
    rows = torch.randn(n, c, generator=g)
    rows *= 10 ** torch.empty(n, 1).uniform_(-2, 1, generator=g)
    rows[:, :D] *= 30
    qn, kn = (1 + 0.4 * torch.randn(D, generator=g) for _ in range(2))
    gain = torch.randn(H, generator=g)
    gain[0] = 0.0
    r = dict(dims=dims, base=300.0)
    at, tot = 13, n + 13
    for p, want in forms_of(rows, dt, dev, g):
        for values in (True, False):
            cache = HybridCache([RunStore(kv=(G, D, V))],
                                n_pages=2 * (tot // 16 + 4), max_slots=3,
                                max_ctx=tot + 32, device=dev, dtype=dt)
            other, slot = cache.alloc_slot(), cache.alloc_slot()
            cache.ensure(slot, tot // 2)
            cache.ensure(other, 20)
            cache.ensure(slot, tot)
            rope = RopeTables(cache.max_ctx, dev)(RopeSpec.from_json(r, True))
            for pool in (cache.key_pool[0], cache.value_pool[0]):
                pool.fill_(3.0)
            norms = ops.HeadNorms(qn.to(dev), kn.to(dev), values,
                                  gain.to(dev) if values else None, eps)
            sl, pos = rows_of(dev, [slot], [n], [tot])
            q = ops.qkv_norm_rope_append(p, norms, cache, 0, w, rope, sl, pos)
            wq, wk, wv = want.split([H * D, G * D, G * V], 1)

            def heads(t, h, weight):
                t = oracle.rms(t.reshape(n, h, D), eps) * f64(weight)
                return oracle.rotate(t, range(at, tot), r)

            wq = heads(wq, H, qn)
            if values:
                wq = wq * f64(gain)[:, None]
            wv = wv.reshape(n, G, V)
            if values:
                wv = oracle.rms(wv, eps)
            lim = tol(dt, 2e-6, 4e-3)
            assert rel(q[..., :D], wq) < lim
            assert bool((q[..., D:] == 0).all())
            pages = cache.page_table[slot, :-(-tot // 16)].long()
            kp, vp = (t[0][pages].transpose(1, 2).flatten(0, 1)
                      for t in (cache.key_pool, cache.value_pool))
            assert rel(kp[at:tot, :, :D], heads(wk, G, kn)) < lim
            assert rel(vp[at:tot, :, :V], wv) < lim
            for t in (kp, vp):
                assert bool((t[:at] == 3).all()) \
                    and bool((t[tot:] == 3).all())
            rest = torch.ones(cache.n_pages + 1, dtype=torch.bool, device=dev)
            rest[pages] = False
            assert bool((cache.key_pool[0][rest] == 3.0).all())
            assert bool((cache.value_pool[0][rest] == 3.0).all())


# --------------------------------------------------------- chunked attention

def soft(H, G, D, V, chunk, dev="cpu", scale=None, sink=True):
    return ops.SoftmaxAttn(H, G, D, V, scale or 1.5 * D ** -0.5,
                           torch.zeros(H, device=dev) if sink else None,
                           chunk=chunk)


def put_kv(cache, w, slot, at, q, k, v):
    """Append rows through the op that neither norms nor rotates."""
    dev, dt = cache.key_pool[0].device, cache.key_pool[0].dtype
    n = q.shape[0]
    cache.ensure(slot, at + n)
    sl, pos = rows_of(dev, [slot], [n], [at + n])
    p = torch.cat([t.reshape(n, -1) for t in (q, k, v)], 1).to(dev, dt)
    still = RopeTables(cache.max_ctx, dev)(RopeSpec(0, 1.0))
    return ops.rope_qkv_append(p, None, cache, 0, w, still, sl, pos), sl, \
        pos, meta_for(dev, [slot], [n], [at + n])


def new_cache(dev, dt, w, kv):
    return HybridCache([RunStore(kv=(w.kv_heads, w.dim, w.vdim))],
                       n_pages=3 * (kv // 16 + 2), max_slots=3,
                       max_ctx=kv + 16, device=dev, dtype=dt)


def o_attention(w, q, k, v, start=0, chunk=None):
    """q [T, H, D], k [N, G, D], v [N, G, V] -> [T, H*V]"""
    R = w.heads // w.kv_heads
    return torch.cat([oracle.chunk_attention(
        f64(q)[:, h], f64(k)[:, h // R], f64(v)[:, h // R], w.scale,
        w.chunk if chunk is None else chunk, start, w.sink is not None)
        for h in range(w.heads)], -1)


@where
@pytest.mark.parametrize("size", [(6, 2, 24, 40), (3, 1, 9, 7),
                                  (20, 1, 64, 136), (8, 2, 128, 128)],
                         ids=str)
@pytest.mark.parametrize("chunk", [1, 48, 64, 100, 1000])
@pytest.mark.parametrize("form", ["whole", "large tiles", "portions",
                                  "single"])
def test_chunked_attention(where, size, chunk, form, monkeypatch):
    """Whole prompts, portions down to two tokens that are cut anywhere in a
    chunk, and single tokens; a gate per head."""
    dev, dt = where
    if form == "large tiles":
        if dev == "cpu":
            pytest.skip("the CPU form has no tiles")
        from ollamamq_amd.ops import hip
        monkeypatch.setattr(hip, "ATTN_LARGE", 0)
    H, G, D, V = size
    kv = 130 if form == "single" else 260
    g = torch.Generator().manual_seed(chunk)
    w = soft(H, G, D, V, chunk, dev, sink=chunk != 64)
    q, k = (torch.randn(kv, h, D, generator=g).to(dt) for h in (H, G))
    v = torch.randn(kv, G, V, generator=g).to(dt)
    z = (2 * torch.randn(kv, H + 3, generator=g)).to(dt)
    cache = new_cache(dev, dt, w, kv)
    other, slot = cache.alloc_slot(), cache.alloc_slot()
    lens = {"whole": [kv], "large tiles": [kv], "single": [1] * kv,
            "portions": [90, 2, 2, 31, 1, 64, 8, 9, 53]}[form]
    got, at = [], 0
    for n in lens:
        cache.ensure(other, min(kv, 40 + at))
        qq, sl, pos, meta = put_kv(cache, w, slot, at, q[at:at + n],
                                   k[at:at + n], v[at:at + n])
        gp = z[at:at + n].to(dev)
        if n <= 2 and dt == BF16 and dev != "cpu":
            gp = ops.Partials(torch.stack([gp.float() - 1, gp * 0 + 1.0]))
        got.append(ops.softmax_attention(
            qq, cache, 0, w, sl, pos, meta, gate=ops.Columns(gp, 3)).cpu())
        at += n
    want = o_attention(w, q, k, v).view(kv, H, V) \
        * oracle.sigmoid(f64(z)[:, 3:])[..., None]
    assert rel(torch.cat(got), want.view(kv, -1)) < tol(dt, 3e-6, 1.2e-2)


def aimed(w, g, kv, marks, dt):
    """Keys at `marks` stand out for every query; all other weights are close
    to zero."""
    k = 0.1 * torch.randn(kv, w.kv_heads, w.dim, generator=g)
    d = torch.randn(w.kv_heads, w.dim, generator=g)
    d /= d.norm(dim=-1, keepdim=True)
    for j in marks:
        k[j] = 4.0 * d
    q = 4.0 * d.repeat_interleave(w.heads // w.kv_heads, 0)
    return q.to(dt), k.to(dt)


def run_at(dev, dt, w, q1, k, v, first, n):
    """The same query n times from position `first` on."""
    cache = new_cache(dev, dt, w, k.shape[0])
    slot = cache.alloc_slot()
    rest = torch.zeros(k.shape[0], w.heads, w.dim)
    put_kv(cache, w, slot, 0, rest, k, v)
    qq = torch.zeros(n, w.heads, cache.key_pool[0].shape[3], dtype=dt)
    qq[..., :w.dim] = q1
    sl, pos = rows_of(dev, [slot], [n], [first + n])
    return ops.softmax_attention(
        qq.to(dev), cache, 0, w, sl, pos,
        meta_for(dev, [slot], [n], [first + n])).cpu()


@where
@pytest.mark.parametrize("chunk", [1, 2, 15, 16, 17, 33, 64, 65, 128, 200])
@pytest.mark.parametrize("n", [1, 2, 40])
def test_chunk_edges(where, chunk, n):
    """A chunk's first key is seen to the chunk's end, the key before it is
    not, wherever a portion begins."""
    dev, dt = where
    H, G, D, V, kv = 4, 2, 32, 24, 290
    g = torch.Generator().manual_seed(3)
    w = soft(H, G, D, V, chunk, dev, scale=1.0)
    starts = {0, chunk - 1, chunk, 2 * chunk - 1, chunk - n, 63, 64, kv - n}
    for first in sorted(s for s in starts if 0 <= s <= kv - n):
        for row in sorted({0, n - 1}):
            lo = (first + row) // chunk * chunk
            q1, k = aimed(w, g, kv, [j for j in (lo - 1, lo) if j >= 0], dt)
            v = torch.randn(kv, G, V, generator=g).to(dt)
            got = run_at(dev, dt, w, q1, k, v, first, n)
            want = o_attention(w, q1.expand(n, H, D), k, v, first)
            assert rel(got, want) < tol(dt, 1e-5, 2e-2), (first, row)
            if lo > 0:
                free = o_attention(w, q1.expand(n, H, D), k, v, first, 0)
                assert rel(free[row], want[row]) > 0.3, "the edge must show"


@where
@pytest.mark.parametrize("n", [1, 2, 40, 300])
def test_far_keys_are_found(where, n):
    """One loud key among hundreds of the same chunk: its first tokens, page,
    step and tile borders."""
    dev, dt = where
    H, G, D, V, kv, chunk = 2, 1, 32, 24, 990, 500
    g = torch.Generator().manual_seed(5)
    w = soft(H, G, D, V, chunk, dev, scale=1.0)
    for j in (500, 501, 511, 512, 527, 528, 576, 639, 640, kv - n):
        q1, k = aimed(w, g, kv, [j], dt)
        v = torch.randn(kv, G, V, generator=g).to(dt)
        got = run_at(dev, dt, w, q1, k, v, kv - n, n)
        want = o_attention(w, q1.expand(n, H, D), k, v, kv - n)
        assert torch.cosine_similarity(want[-1, :V], f64(v[j, 0]), 0) > 0.9
        assert rel(got, want) < tol(dt, 1e-5, 2e-2), j


@where
@pytest.mark.parametrize("n", [1, 40])
def test_one_in_the_denominator(where, n):
    """Scores far below zero leave almost nothing, scores far above do not
    notice; the sum is over the query's chunk only."""
    dev, dt = where
    H, G, D, V, kv = 4, 2, 32, 24, 90
    g = torch.Generator().manual_seed(9)
    w = soft(H, G, D, V, 60, dev, scale=2.0)
    q1, k = aimed(w, g, kv, [70], dt)            # one score of 32
    v = torch.randn(kv, G, V, generator=g).to(dt)
    for scale in (2.0, 0.01, -0.01):
        w = w._replace(scale=scale)
        want = o_attention(w, q1.expand(n, H, D), k, v, kv - n)
        got = run_at(dev, dt, w, q1, k, v, kv - n, n)
        assert rel(got, want) < tol(dt, 1e-5, 2e-2)
    alone = k[70:71].expand(kv, G, D).contiguous()
    w = w._replace(scale=-2.0)
    got = run_at(dev, dt, w, q1, alone, v, kv - n, n)
    assert got.abs().max() < 1e-9


# ----------------------------------------------------------------- retention

def retention_case(dev, dt, H, D, V, decay, n, seed=0):
    g = torch.Generator().manual_seed(seed)
    w = ops.LightningWeights(
        H, D, V, (0, H * D, 2 * H * D, 2 * H * D + H * V),
        ops.decay_powers(decay, dev), None, 1e-2, act=False,
        scale=D ** -0.5, per_head=True, gate="silu")
    p = torch.randn(n, 2 * H * (D + V), generator=g)
    p[:, 2 * H * D:2 * H * D + V] *= 5           # a head far from the others
    return g, w, p.to(dt)


def o_retention(w, p, decay):
    H, D, V = w.heads, w.dim, w.vdim
    n = p.shape[0]
    q, k, v, gate = f64(p).split([H * D, H * D, H * V, H * V], 1)
    o, S = oracle.retention_heads(q.view(n, H, D),
                                  k.view(n, H, D) * D ** -0.5,
                                  v.view(n, H, V), decay)
    return oracle.rms(o, w.eps).reshape(n, -1) * oracle.silu(gate), S


def feed(op, p, lens, dev, dt, slot=1):
    """Call op(rows, slots, positions, meta) for portions of p."""
    got, at = [], 0
    for m in lens:
        sl, pos = rows_of(dev, [slot], [m], [at + m])
        pd = p[at:at + m].to(dev)
        if m < 3 and dt == BF16 and dev != "cpu":
            pd = ops.Partials(torch.stack([pd.float() - 1, pd * 0 + 1.0]))
        got.append(op(pd, sl, pos, meta_for(dev, [slot], [m], [at + m]))
                   .cpu())
        at += m
    return torch.cat(got)


FORMS = {"whole": [210], "single": [1] * 75,
         "portions": [70, 2, 3, 1, 64, 5, 65]}
forms = pytest.mark.parametrize("form", list(FORMS))


@where
@pytest.mark.parametrize("size", [(3, 24, 40), (2, 9, 7), (4, 64, 64),
                                  (2, 128, 128), (1, 200, 136), (1, 300, 16),
                                  (2, 16, 300)], ids=str)
@forms
def test_retention(where, size, form):
    """A dirty slot is taken as empty at position 0 and carried after that;
    chunks, token by token and portions of both agree."""
    dev, dt = where
    H, D, V = size
    decay, lens = [0.999, 0.3, 0.9, 0.0][:H], FORMS[form]
    g, w, p = retention_case(dev, dt, H, D, V, decay, sum(lens))
    state = torch.full((3, H, D, V), 7.0, device=dev)
    got = feed(lambda x, sl, pos, m: ops.lightning(x, w, state, sl, pos, m),
               p, lens, dev, dt)
    want, S = o_retention(w, p, decay)
    assert rel(got, want) < tol(dt, 5e-6, 1e-2)
    assert rel(state[1] * w.scale, S) < tol(dt, 5e-6, 5e-3)
    assert bool((state[0] == 7).all()) and bool((state[2] == 7).all())


# --------------------------------------------------------------- delta rules

def gated_case(dev, dt, H, G, D, V, taps, n, seed=0, rate=0.0, ranks=(8, 16),
               bias=-2.0):
    """rate: the mean of the decays' logarithmic rates."""
    g = torch.Generator().manual_seed(seed)
    r = lambda *s: torch.randn(*s, generator=g)
    C = 2 * G * D + H * V
    at = -(-(C + H) // 8) * 8
    offsets = (0, C, at, at + ranks[0])
    t = dict(conv=1.5 * r(C, taps) / taps ** 0.5,
             a2=(r(H * D, ranks[0]) / ranks[0] ** 0.5).to(BF16),
             A_log=rate + 0.5 * r(H), dt_bias=bias + r(H * D),
             g2=(r(H * V, ranks[1]) / ranks[1] ** 0.5).to(BF16),
             norm=1 + 0.3 * r(V))
    put = lambda x: x.to(dev, dt).contiguous()
    w = ops.GatedDeltaWeights(
        H, G, D, V, offsets, t["conv"].t().contiguous().to(dev),
        ops.low_rank(put(t["a2"])), t["A_log"].exp().to(dev),
        t["dt_bias"].to(dev), ops.low_rank(put(t["g2"])),
        t["norm"].to(dev), 1e-4)
    p = r(n, offsets[3] + ranks[1] + 8 - ranks[1] % 8).to(dt)
    return g, w, t, p


def o_gated(w, t, p, parts=False):
    H, G, D, V = w.heads, w.kv_heads, w.dim, w.vdim
    o_in, ob, oa, og = w.offsets
    n, x = p.shape[0], f64(p)
    C = w.conv.shape[1]
    t = {k: f64(v) for k, v in t.items()}
    y = oracle.silu(oracle.short_conv(x[:, o_in:o_in + C], t["conv"]))
    q, k, v = y.split([G * D, G * D, H * V], 1)
    R = H // G
    q = (oracle.unit(q.view(n, G, D)) * D ** -0.5).repeat_interleave(R, 1)
    k = oracle.unit(k.view(n, G, D)).repeat_interleave(R, 1)
    z = x[:, oa:oa + w.a2.rank] @ t["a2"].T + t["dt_bias"]
    g = torch.exp(-torch.exp(t["A_log"])[None, :, None]
                  * oracle.softplus(z).view(n, H, D))
    o, S = oracle.gated_delta_heads(q, k, v.view(n, H, V), g,
                                    oracle.sigmoid(x[:, ob:ob + H]))
    gate = oracle.sigmoid(x[:, og:og + w.g2.rank] @ t["g2"].T)
    o = (oracle.rms(o, w.eps) * t["norm"]).reshape(n, H * V) * gate
    return o, S, x[:, o_in:o_in + C]


def gated_run(w, state, conv):
    return lambda x, sl, pos, m: ops.gated_delta(x, w, state, conv, sl, pos,
                                                 m)


GATED = [(4, 2, 16, 24, 4), (2, 2, 9, 7, 3), (3, 1, 64, 64, 4),
         (2, 1, 128, 128, 4), (1, 1, 200, 136, 2), (1, 1, 300, 16, 4),
         (2, 2, 24, 300, 1), (6, 3, 32, 40, 20)]


@where
@pytest.mark.parametrize("size", GATED, ids=str)
@forms
def test_gated_delta(where, size, form):
    """Groups of heads that share a key, one to many taps, inputs of the
    convolution from before the portion, dirty slots."""
    dev, dt = where
    H, G, D, V, taps = size
    lens = FORMS[form]
    g, w, t, p = gated_case(dev, dt, *size, sum(lens))
    state = torch.full((3, H, D, V), 7.0, device=dev)
    conv = torch.full((3, taps - 1, w.conv.shape[1]), 5.0, device=dev)
    got = feed(gated_run(w, state, conv), p, lens, dev, dt)
    want, S, x = o_gated(w, t, p)
    assert rel(got, want) < tol(dt, 2e-5, 1.5e-2)
    assert rel(state[1], S) < tol(dt, 2e-5, 1e-2)
    if taps > 1:
        assert rel(conv[1], x[1 - taps:]) < tol(dt, 1e-6, 1e-6)
    for s, fill in ((state, 7), (conv, 5)):
        assert bool((s[0] == fill).all()) and bool((s[2] == fill).all())


@where
@pytest.mark.parametrize("rate,bias", [(-6.0, -2.0), (0.0, -2.0),
                                       (1.0, 1.0), (2.0, 1.5), (5.0, 1.0),
                                       (8.0, -3.0)])
@pytest.mark.parametrize("D", [32, 96])
def test_gated_delta_decays(where, rate, bias, D):
    """From almost none to all within a token, channels of both kinds side by
    side."""
    dev, dt = where
    lens = [140, 1, 1, 3, 65]
    g, w, t, p = gated_case(dev, dt, 2, 1, D, 40, 4, sum(lens), rate=rate,
                            bias=bias)
    t["dt_bias"][::3] = -9.0                     # these remember
    w = w._replace(dt_bias=t["dt_bias"].to(dev))
    state = torch.full((2, 2, D, 40), 7.0, device=dev)
    conv = torch.zeros(2, 3, w.conv.shape[1], device=dev)
    got = feed(gated_run(w, state, conv), p, lens, dev, dt)
    want, S, _ = o_gated(w, t, p)
    assert rel(got, want) < tol(dt, 4e-5, 1.5e-2)
    assert rel(state[1], S) < tol(dt, 4e-5, 1e-2)


@where
@pytest.mark.parametrize("taps", [1, 2, 4, 5, 18])
def test_short_convolution_edges(where, taps):
    """Each place in a portion reads the right inputs: one loud input shows
    for exactly `taps` tokens, across portions of every size."""
    dev, dt = where
    lens = [3, 1, 2, 17, 1, 1, 33, 5, 16, 1]
    n = sum(lens)
    for loud in (0, 2, 3, 5, 22, 24, 57, n - 1):
        g, w, t, p = gated_case(dev, dt, 2, 1, 8, 16, taps, n, seed=loud)
        C = w.conv.shape[1]
        p[:, :C] *= 0.01
        p[loud, :C] = (6 * torch.randn(C, generator=g)).to(dt)
        state = torch.zeros(2, 2, 8, 16, device=dev)
        conv = torch.full((2, taps - 1, C), 9.0, device=dev)
        got = feed(gated_run(w, state, conv), p, lens, dev, dt)
        want, S, _ = o_gated(w, t, p)
        assert rel(got[loud:loud + taps], want[loud:loud + taps]) \
            < tol(dt, 2e-5, 1.5e-2), loud
        assert rel(got, want) < tol(dt, 5e-5, 2e-2), loud


def general_case(dev, dt, H, D, n, seed=0, rank=16):
    g = torch.Generator().manual_seed(seed)
    r = lambda *s: torch.randn(*s, generator=g)
    N = H * D
    at = -(-5 * N // 8) * 8
    t = dict(w2=(2 * r(N, rank) / rank ** 0.5).to(BF16), w0=-1 + 1.5 * r(N),
             a_bias=r(N), norm=1 + 0.3 * r(N))
    w = ops.GeneralDeltaWeights(
        H, D, (0, N, 2 * N, 3 * N, 4 * N, at),
        ops.low_rank(t["w2"].to(dev, dt).contiguous()), t["w0"].to(dev),
        t["a_bias"].to(dev), t["norm"].to(dev), 1e-4)
    p = r(n, at + rank + 8)
    p[:, N:2 * N] *= 0.4
    return g, w, t, p.to(dt)


def o_general(w, t, p):
    H, D = w.heads, w.dim
    N, n, x = H * D, p.shape[0], f64(p)
    t = {k: f64(v) for k, v in t.items()}
    r, k, v, a, gate = x[:, :5 * N].split(N, 1)
    at = w.offsets[5]
    z = torch.tanh(x[:, at:at + w.w2.rank]) @ t["w2"].T + t["w0"]
    decay = torch.exp(-math.exp(-0.5) * oracle.sigmoid(z))
    hd = lambda y: y.reshape(n, H, D)
    o, S = oracle.general_delta_heads(hd(r), hd(k), hd(v), hd(decay),
                                      oracle.sigmoid(hd(a + t["a_bias"])))
    return oracle.rms(o, w.eps).reshape(n, N) * t["norm"] \
        * oracle.sigmoid(gate), S


def general_run(w, state):
    return lambda x, sl, pos, m: ops.general_delta(x, w, state, sl, pos, m)


@where
@pytest.mark.parametrize("size", [(5, 16), (3, 10), (2, 64), (1, 128),
                                  (1, 200), (1, 300), (4, 7)], ids=str)
@forms
def test_general_delta(where, size, form):
    dev, dt = where
    H, D = size
    lens = FORMS[form]
    g, w, t, p = general_case(dev, dt, H, D, sum(lens),
                              rank=8 if D == 10 else 40)
    state = torch.full((3, H, D, D), 7.0, device=dev)
    got = feed(general_run(w, state), p, lens, dev, dt)
    want, S = o_general(w, t, p)
    assert rel(got, want) < tol(dt, 2e-5, 1.5e-2)
    assert rel(state[1], S) < tol(dt, 2e-5, 1e-2)
    assert bool((state[0] == 7).all()) and bool((state[2] == 7).all())


@where
def test_general_delta_keys(where):
    """Removal goes along the unit key whatever its length: keys from far
    below the eps to large, the same key again and again."""
    dev, dt = where
    H, D, lens = 2, 32, [100, 1, 2, 30]
    n = sum(lens)
    g, w, t, p = general_case(dev, dt, H, D, n)
    N = H * D
    size = torch.logspace(-5, 0.3, n)[torch.randperm(n, generator=g)]
    p[:, N:2 * N] = (torch.randn(1, N, generator=g) * size[:, None]).to(dt)
    state = torch.zeros(2, H, D, D, device=dev)
    got = feed(general_run(w, state), p, lens, dev, dt)
    want, S = o_general(w, t, p)
    assert rel(got, want) < tol(dt, 5e-5, 2e-2)
    assert rel(state[1], S) < tol(dt, 5e-5, 1e-2)


@where
@pytest.mark.parametrize("n", [1, 2, 63, 64, 65, 150])
@pytest.mark.parametrize("rule", ["gated", "general", "retention"])
def test_far_tokens_are_remembered(where, rule, n):
    """One loud token long ago is what the last query returns, at chunk
    borders and from before the portion."""
    dev, dt = where
    H, D, V, kv = 2, 32, 32, 400
    for j in (0, 63, 64, 128, 200, kv - n):
        if rule == "gated":
            g, w, t, p = gated_case(dev, dt, H, H, D, V, 1, kv, seed=j,
                                    rate=-9.0)
            ahead, C = H * D, w.conv.shape[1]
            want_of = lambda x: o_gated(w, t, x)[0]
        elif rule == "general":
            g, w, t, p = general_case(dev, dt, H, D, kv, seed=j)
            t["w0"].fill_(-12.0)                 # decays of almost one
            w = w._replace(w0=t["w0"].to(dev))
            p[:, w.offsets[5]:] *= 0.01
            ahead, C = H * D, 3 * H * D
            want_of = lambda x: o_general(w, t, x)[0]
        else:
            g, w, p = retention_case(dev, dt, H, D, V, [1.0, 0.9995], kv, j)
            ahead, C = H * D, 2 * H * D + H * V
            want_of = lambda x: o_retention(w, x, [1.0, 0.9995])[0]
        x = p.clone()
        x[:, :C] *= 0.02
        if rule == "gated":
            x[:, C:C + H] = -9.0                 # steps of almost nothing
            x[j, C:C + H] = 3.0
        x[j, ahead:C] = (1 + torch.randn(C - ahead, generator=g)).to(dt)
        x[-1, :ahead] = 2.0
        state = torch.full((2, H, D, V), -3.0, device=dev)
        conv = torch.zeros(2, 0, w.conv.shape[1], device=dev) \
            if rule == "gated" else None
        op = gated_run(w, state, conv) if rule == "gated" \
            else general_run(w, state) if rule == "general" \
            else lambda y, sl, pos, m: ops.lightning(y, w, state, sl, pos, m)
        lens = [kv - n, n] if n < kv else [n]
        got = feed(op, x, lens, dev, dt)
        want = want_of(x)
        gone = x.clone()
        gone[j, ahead:C] = 0
        assert rel(want_of(gone)[-1:], want[-1:]) > 0.3, "it must show"
        assert rel(got[-1:], want[-1:]) < tol(dt, 5e-5, 2e-2), j


@where
@pytest.mark.parametrize("rule", ["gated", "general", "retention"])
@pytest.mark.parametrize("held", [1, 3, 1 << 20])
def test_recurrent_batch(where, rule, held, monkeypatch):
    """Single tokens, short and long portions of several slots in one call,
    the chunks' factors held a few or all at a time."""
    dev, dt = where
    H, D, V = 2, 24, 40 if rule != "general" else 24
    if dev != "cpu":
        from ollamamq_amd.ops import hip
        one = 4 * hip._lib.delta_scratch_floats(int(rule == "general"), 1, H,
                                                D)
        monkeypatch.setattr(hip, "DELTA_BYTES", held * one)
    elif held != 1:
        pytest.skip("the CPU form holds nothing")
    lens, before = [1, 1, 3, 70, 200, 130], [40, 0, 5, 64, 0, 2]
    make = {"gated": lambda n, i: gated_case(dev, dt, H, 1, D, V, 4, n, i),
            "general": lambda n, i: general_case(dev, dt, H, D, n, i),
            "retention": lambda n, i: retention_case(
                dev, dt, H, D, V, [0.98, 0.7], n, i)}[rule]
    cases = [make(b + n, i) for i, (n, b) in enumerate(zip(lens, before))]
    w = cases[0][1]
    state = torch.full((7, H, D, V), 9.0, device=dev)
    conv = torch.full((7, 3, 2 * D + H * V), 9.0, device=dev)
    op = {"gated": gated_run(w, state, conv), "general": general_run(w, state),
          "retention": lambda y, sl, pos, m: ops.lightning(
              y, w, state, sl, pos, m)}[rule]
    ref = {"gated": lambda p: o_gated(w, cases[0][2], p)[0],
           "general": lambda p: o_general(w, cases[0][2], p)[0],
           "retention": lambda p: o_retention(w, p, [0.98, 0.7])[0]}[rule]
    slots = [3, 0, 5, 1, 2, 6]
    for s, c, b in zip(slots, cases, before):
        if b:
            feed(op, c[-1], [b], dev, dt, s)
    tot = [b + n for b, n in zip(before, lens)]
    sl, pos = rows_of(dev, slots, lens, tot)
    got = op(torch.cat([c[-1][b:] for c, b in zip(cases, before)]).to(dev),
             sl, pos, meta_for(dev, slots, lens, tot, n_decode=2)).cpu()
    for c, b, part in zip(cases, before, got.split(lens)):
        assert rel(part, ref(c[-1])[b:]) < tol(dt, 2e-5, 1.5e-2)


@GPU
@pytest.mark.parametrize("users", [1, 40, 64])
@pytest.mark.parametrize("D", [32, 64])
def test_fused_step(users, D):
    """Decode steps of many sequences norm and gate in the same kernel, few
    in their own; rows and fragment layout."""
    H, dev, dt = 16, "cuda:0", BF16
    g, w, t, p = general_case(dev, dt, H, D, 3 * users, seed=users)
    eye = torch.eye(H * D, dtype=BF16, device=dev)
    packed = ops.pack_weight(eye)
    for frag in (False, True):
        state = torch.zeros(users + 1, H, D, D, device=dev)
        got = []
        for i in range(3):
            sl, pos = rows_of(dev, list(range(users)), [1] * users,
                              [i + 1] * users)
            o = ops.general_delta(p[i::3].to(dev), w, state, sl, pos, meta_for(
                dev, list(range(users)), [1] * users, [i + 1] * users), frag)
            got.append((ops.linear(o, eye, packed=packed) if frag else o)
                       .cpu())
        got = torch.stack(got, 1)
        for u in range(0, users, 13):
            want = o_general(w, t, p[3 * u:3 * u + 3])[0]
            assert rel(got[u], want) < 1.5e-2


# --------------------------------------------------------------- whole models

def test_config_reaches_every_constant(models):
    pc = PemidraConfig.from_json(models["mixed"][1])
    assert (pc.eps, pc.alpha) == (1e-5, 1.7)
    a, b, c, d, e = pc.layers
    assert a.mixer.decay == (0.3, 0.9, 0.995) and a.ff == 80
    left, right = b.mixer.left, b.mixer.right
    assert (left.heads, left.kv_heads, left.dim, left.vdim, left.chunk,
            left.scale) == (6, 2, 24, 40, 37, 0.3)
    assert left.rope == RopeSpec(8, 500.0, None, True) and b.ff is None
    assert (right.heads, right.kv_heads, right.dim, right.vdim,
            right.conv) == (4, 2, 16, 24, 3)
    assert (c.mixer.heads, c.mixer.dim, c.ff) == (5, 16, 96)
    stores = pc.run_stores()
    assert stores[0].state == (("retention", (3, 24, 40)),)
    assert stores[1].kv == (2, 24, 40)
    assert stores[1].state == (("delta", (4, 16, 24)),
                               ("conv", (2, 2 * 2 * 16 + 4 * 24)))
    assert stores[2].state == (("delta", (5, 16, 16)),)


@exact
@pytest.mark.parametrize("name", list(MODELS))
def test_every_layer(models, where, name):
    """The residual stream after every layer."""
    dev, dt = where
    path, cfg, w = models[name]
    toks = tokens_for(name, 40)
    _, want = oracle.run(cfg, w, toks)
    pc = config_from_folder(path)
    model = build_model(pc, device=dev, dtype=dt)
    kv = cache_for_model(pc, n_pages=8, max_slots=2, max_ctx=64, device=dev,
                         dtype=dt)
    slot = kv.alloc_slot()
    kv.ensure(slot, 40)
    sl, pos = rows_of(dev, [slot], [40], [40])
    out = []
    model.forward(torch.tensor(toks, dtype=torch.int32, device=dev), pos, kv,
                  sl, meta_for(dev, [slot], [40], [40]), layer_out=out)
    assert len(out) == len(want) == len(pc.layers)
    for got, ref in zip(out, want):
        assert got.dtype == F32 and rel(got, ref) < 2e-5


@where
@pytest.mark.parametrize("name", list(MODELS))
def test_prompt(models, where, name):
    dev, dt = where
    toks = tokens_for(name, 140)
    eng = make_engine(models[name][0], dt, 192, dev)
    check(run_portions(eng, toks, [140]), expected(models, name, toks), dt)


@where
@pytest.mark.parametrize("name", list(MODELS))
@pytest.mark.parametrize("size", [1, 2, 3, 17, 64, 65])
def test_portions_agree_with_the_whole(models, where, name, size):
    dev, dt = where
    toks = tokens_for(name, 140)
    eng = make_engine(models[name][0], dt, 192, dev)
    check(run_portions(eng, toks, cut(140, size)),
          expected(models, name, toks), dt)


@where
@pytest.mark.parametrize("name", ["mixed", "odd", "packed"])
def test_mixed_batches_and_reused_memory(models, where, name):
    """Four slots and just enough pages, seven requests of unequal length:
    prompts' portions beside decoded tokens, pauses, freed pages and slots
    taken over by the next request."""
    dev, dt = where
    g = torch.Generator().manual_seed(4)
    reqs = [tokens_for(name, n, i) for i, n in
            enumerate((90, 1, 33, 17, 64, 2, 50))]
    eng = make_engine(models[name][0], dt, 96 + 48 + 64 + 64, dev)
    waiting, live, got = list(range(7)), {}, {i: [] for i in range(7)}
    at = [0] * 7
    while waiting or live:
        while waiting and len(live) < 4 and (
                len(live) < 3 or eng.kv.free_page_count() >= 6):
            i = waiting.pop(0)
            live[i] = eng.open_stream()
        parts, who = [], []
        for i, s in live.items():
            if torch.rand((), generator=g) < 0.2 and len(live) > 1:
                continue                                  # left out this time
            left = len(reqs[i]) - at[i]
            n = min(left, [1, 1, 2, 5, 16, 31][
                int(torch.randint(0, 6, (), generator=g))])
            parts.append((s, reqs[i][at[i]:at[i] + n], list(range(n))))
            who.append((i, n))
        if not parts:
            continue
        out = eng.feed(parts).cpu()
        for i, n in who:
            got[i].append(out[:n])
            out = out[n:]
            at[i] += n
            if at[i] == len(reqs[i]):
                eng.close_stream(live.pop(i))
    for i, toks in enumerate(reqs):
        check(torch.cat(got[i]), expected(models, name, toks), dt)
    assert eng.kv.free_page_count() == eng.kv.n_pages


@where
@pytest.mark.parametrize("name", ["mixed", "packed"])
def test_long_decoding(models, where, name):
    """Chunk after chunk passes over decoded tokens."""
    dev, dt = where
    toks = tokens_for(name, 300)
    eng = make_engine(models[name][0], dt, 320, dev)
    got = run_portions(eng, toks, [7] + [1] * 293)
    check(got[200:], expected(models, name, toks)[200:], dt)


@where
@pytest.mark.parametrize("name", ["mixed", "packed"])
def test_batch_neighbours_do_not_matter(models, where, name):
    """A stream's logits beside others are those it has alone."""
    dev, dt = where
    toks, noise = tokens_for(name, 70), tokens_for(name, 70, 9)
    want = run_portions(make_engine(models[name][0], dt, 256, dev), toks,
                        [40, 1, 2, 20, 1, 1, 5])
    eng = make_engine(models[name][0], dt, 256, dev)
    a, b, c = (eng.open_stream() for _ in range(3))
    got, at = [], 0
    for i, n in enumerate([40, 1, 2, 20, 1, 1, 5]):
        other = [(b, noise[2 * i:2 * i + 2], []),
                 (c, noise[i:i + 1], [0])]
        out = eng.feed([other[1], (a, toks[at:at + n], list(range(n))),
                        other[0]])
        got.append(out[1:].cpu())
        at += n
    check(torch.cat(got), want.to(F64), dt)


@where
def test_first_tokens(models, where):
    """Sequences of one to three tokens, decoded from nothing and
    prefilled."""
    dev, dt = where
    for name in MODELS:
        toks = tokens_for(name, 3)
        want = expected(models, name, toks)
        for cuts in ([1, 1, 1], [2, 1], [3], [1, 2]):
            eng = make_engine(models[name][0], dt, 64, dev)
            check(run_portions(eng, toks, cuts), want, dt)


@exact
@pytest.mark.parametrize("name", ["mixed", "odd", "packed"])
def test_greedy_generation(models, where, name):
    """Through submit/step: admission, chunked prompts, mixed steps, the
    pipelined decode, slots that are freed and taken again.  Every token is
    the oracle's argmax (or a tie within rounding)."""
    dev, dt = where
    path, cfg, w = models[name]
    pc = config_from_folder(path)
    kv = cache_for_model(pc, n_pages=40, max_slots=3, max_ctx=160,
                         device=dev, dtype=dt)
    eng = LlamaEngine(build_model(pc, device=dev, dtype=dt), kv, max_batch=3,
                      prefill_chunk=24)
    prompts = [tokens_for(name, n, i) for i, n in enumerate((5, 61, 1, 30))]
    out = generate(eng, prompts, 12)
    for p, o in zip(prompts, out):
        assert len(o) == 12
        lg = oracle.run(cfg, w, p + o[:-1])[0][len(p) - 1:]
        for step, tok in zip(lg, o):
            assert step.max() - step[tok] < 1e-4
    assert kv.free_page_count() == 40


@GPU
@pytest.mark.parametrize("name,dt", [("mixed", F32), ("packed", BF16)])
def test_graph_replay_equals_eager(models, name, dt):
    """Captured decode with batch padding and host work between replays
    against the same steps without graphs."""
    path = models[name][0]
    pc = config_from_folder(path)

    def run(graphs):
        kv = cache_for_model(pc, n_pages=64, max_slots=6, max_ctx=160,
                             device="cuda:0", dtype=dt)
        eng = LlamaEngine(build_model(pc, device="cuda:0", dtype=dt), kv,
                          max_batch=6)
        assert eng.model.frag_decode == (dt == BF16)
        eng.use_graphs = eng.use_pipeline = graphs
        if graphs:
            eng.warm_graphs()
        return generate(eng, [tokens_for(name, n, n) for n in
                              (3, 20, 9, 14, 30)], 25)

    assert run(True) == run(False)


@GPU
@pytest.mark.parametrize("users", [1, 33, 64])
def test_decode_batches(models, users):
    """Batches of one and of more than one half of the fragment layout."""
    path = models["packed"][0]
    pc = config_from_folder(path)
    kv = cache_for_model(pc, n_pages=users * 4, max_slots=users, max_ctx=64,
                         device="cuda:0", dtype=BF16)
    eng = LlamaEngine(build_model(pc, device="cuda:0", dtype=BF16), kv,
                      max_batch=users)
    streams = [eng.open_stream() for _ in range(users)]
    toks = [tokens_for("packed", 6, u % 5) for u in range(users)]
    got = torch.stack([eng.feed([(s, t[i:i + 1], [0])
                                 for s, t in zip(streams, toks)]).cpu()
                       for i in range(6)], 1)
    for u in range(users):
        check(got[u], expected(models, "packed", toks[u]), BF16)


@where
def test_preset_runs(where):
    dev, dt = where
    from ollamamq_amd.models import PRESETS
    cfg = PRESETS["pemidra-tiny"]
    kv = cache_for_model(cfg, n_pages=32, max_slots=2, max_ctx=128,
                         device=dev, dtype=dt)
    model = build_model(cfg, device=dev, dtype=dt, seed=3)
    assert model.weight_bytes() > 0 and cfg.weight_bytes() > 0
    eng = LlamaEngine(model, kv, max_batch=2)
    out = generate(eng, [[1, 2, 3], [4] * 20], 5)
    assert all(len(o) == 5 for o in out)
    h = torch.tensor(eng.embed([1, 2, 3]), dtype=F64)
    z = (h - f64(model.final_norm.b)) / f64(model.final_norm.w)
    assert len(h) == cfg.width and abs(z.pow(2).mean() - 1) < 0.05
    assert cfg.model_info()["block_count"] == 4


# ------------------------------------------------------------ loading, runner

def test_bad_checkpoints_are_refused(models, tmp_path):
    path, cfg, w = models["odd"]
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    bad = dict(w)
    bad["l0.mix.right.dt_bias"] = torch.zeros(3, dtype=BF16)
    save_file(bad, str(tmp_path / "model.safetensors"))
    with pytest.raises(ValueError, match="l0.mix.right.dt_bias"):
        build_model(config_from_folder(str(tmp_path)))
    del bad["l0.mix.right.dt_bias"]
    save_file(bad, str(tmp_path / "model.safetensors"))
    with pytest.raises(KeyError, match="l0.mix.right.dt_bias"):
        build_model(config_from_folder(str(tmp_path)))

    def changed(i, mixer=None, side=None, **kw):
        other = json.loads(json.dumps(cfg))
        other["layers"][i].update(kw)
        m = other["layers"][i]["mixer"]
        (m[side] if side else m).update(mixer or {})
        return PemidraConfig.from_json(other)

    with pytest.raises(ValueError, match="something"):
        changed(0, type="something")
    with pytest.raises(ValueError, match="moe"):
        changed(0, mlp={"kind": "moe", "ff": 3})
    with pytest.raises(ValueError, match="2 decays"):
        changed(1, {"decay": [0.5, 0.5]})
    with pytest.raises(ValueError, match="evenly"):
        changed(0, {"kv_heads": 2}, "left")
    with pytest.raises(ValueError, match="evenly"):
        changed(0, {"kv_heads": 2}, "right")
    with pytest.raises(ValueError, match="10 rotated"):
        changed(0, {"rot": {"dims": 10, "base": 10.0}}, "left")
    with pytest.raises(ValueError, match="3 rotated"):
        changed(0, {"rot": {"dims": 3, "base": 10.0}}, "left")
    with pytest.raises(ValueError, match="chunks of 0"):
        changed(0, {"mask": {"size": 0}}, "left")
    with pytest.raises(ValueError, match="0 taps"):
        changed(0, {"conv": 0}, "right")
    with pytest.raises(ValueError, match="parallel"):
        build_model(PemidraConfig.from_json(cfg), tp_size=2)


@exact
def test_trace_runner(models, where, tmp_path):
    dev, _ = where
    path = models["mixed"][0]
    a, b = tokens_for("mixed", 50), tokens_for("mixed", 20, 1)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:41], "want": [40]}],
         "end": []},
        {"step": 1, "entries": [{"id": "b", "tokens": b[:7], "want": [0, 6]},
                                {"id": "a", "tokens": a[41:42],
                                 "want": []}], "end": []},
        {"step": 2, "entries": [{"id": "b", "tokens": b[7:8], "want": []}],
         "end": []},
        {"step": 3, "entries": [{"id": "b", "tokens": b[8:], "want": [11]},
                                {"id": "a", "tokens": a[42:],
                                 "want": [7, 3]}], "end": ["a", "b"]},
        {"step": 4, "entries": [{"id": "a", "tokens": b, "want": [5]}],
         "end": ["a"]},
    ]
    p = subprocess.run(
        [os.path.join(REPO, "bin", "trace_run"), "--model", path, "--dtype",
         "float32", "--out", str(tmp_path), "--max-tokens", "128",
         "--device", dev], input="".join(json.dumps(s) + "\n"
                                         for s in steps),
        capture_output=True, text=True, timeout=240)
    assert p.returncode == 0, p.stderr[-2000:]
    done = [x for x in p.stdout.splitlines() if x.startswith("done")]
    assert done == [f"done {i}" for i in range(5)]

    def read(i):
        data = (tmp_path / f"{i}.f32").read_bytes()
        return torch.frombuffer(bytearray(data), dtype=F32).view(-1, 200)
    ea, eb = expected(models, "mixed", a), expected(models, "mixed", b)
    check(read(0), ea[[40]], F32)
    check(read(1), eb[[0, 6]], F32)
    assert not (tmp_path / "2.f32").exists()
    check(read(3), torch.stack([eb[19], ea[49], ea[45]]), F32)
    check(read(4), eb[[5]], F32)


def test_worker_serves_a_checkpoint(models):
    import queue
    from ollamamq_amd.engine.worker import Worker
    from ollamamq_amd.models import PRESETS, register_checkpoint
    if torch.cuda.is_available():
        pytest.skip("CPU form of the worker test")
    register_checkpoint(f"pemidra-folder={models['mixed'][0]}")
    try:
        w = Worker(0, max_batch=2, default_ctx=128)
        assert "pemidra-folder" in w.available_models()
        q = queue.Queue()
        w.generate("pemidra-folder", [1, 2, 3], GenParams(max_tokens=6),
                   lambda t, done: q.put((t, done)))
        out = []
        while True:
            t, done = q.get(timeout=60)
            if done:
                break
            out.append(t)
        assert len(out) == 6
        assert w.unload("pemidra-folder") is None
    finally:
        PRESETS.pop("pemidra-folder")
