"""The Kavedra design against a plain float64 statement of its equations
(kavedra_oracle.py): every mechanism alone, then whole models fed in
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

import kavedra_oracle as oracle
from hybrid_common import (BF16, F32, F64, GPU, cut, exact, generate,
                           meta_for, rel, rows_of, run_portions, tol, where)
from ollamamq_amd.engine import (GenParams, HybridCache, LlamaEngine,
                                 cache_for_model)
from ollamamq_amd.engine.kvcache import RunStore
from ollamamq_amd.engine.trace import make_engine
from ollamamq_amd.models import (KavedraConfig, build_model,
                                 config_from_folder)
from ollamamq_amd.models.hybrid import RopeSpec, RopeTables
from ollamamq_amd.ops import interface as ops

REPO = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def rot(dims, base=1e4, yarn=None):
    """yarn: (factor, original, fast, slow)"""
    d = {"dims": dims, "base": base}
    if yarn:
        d["scaling"] = dict(zip(("factor", "original", "fast", "slow"), yarn))
    return d


def layer(kind, ff, **mixer):
    return {"type": kind, "mixer": mixer,
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def light(heads, dim, vdim, decay, ff=None):
    return layer("lightning", ff, heads=heads, dim=dim, vdim=vdim,
                 decay=decay)


def attn(heads, kv_heads, dim, vdim, r, ff=None, scale=None):
    return layer("attention", ff, heads=heads, kv_heads=kv_heads, dim=dim,
                 vdim=vdim, rot=r, scale=scale or dim ** -0.5)


def latent(heads, dim, vdim, rank, r, window, ff=None, scale=None):
    return layer("latent_attention", ff, heads=heads, dim=dim, vdim=vdim,
                 kv_rank=rank, rot=r, rot_dim=r["dims"],
                 mask={"size": window} if window else None,
                 scale=scale or (dim + r["dims"]) ** -0.5)


def config(width, vocab, layers, loop=None, eps=1e-5, scale=1.5):
    return {"architecture": "Kavedra", "width": width, "vocab": vocab,
            "layers": layers, "norm": {"eps": eps}, "logit_scale": scale,
            "loop": dict(zip(("start", "stop", "times"), loop))
            if loop else None}


MODELS = {
    # no two layers alike, some without a feed-forward, a loop in the middle
    "mixed": config(128, 200, [
        light(3, 24, 40, [0.3, 0.9, 0.995], 80),
        latent(5, 16, 24, 56, rot(8, 500.0, (4.0, 64, 8.0, 1.0)), 37, 96),
        attn(6, 2, 24, 40, rot(8)),
        light(2, 16, 72, [0.97, 0.5]),
        latent(2, 40, 16, 24, rot(24), 100, 72)], loop=(1, 4, 2)),
    # sizes that fit no tile, windows of one token and of all, a loop that
    # starts with the first layer, nothing rotated
    "odd": config(90, 131, [
        light(3, 9, 7, [0.0, 1.0, 0.8], 34),
        attn(3, 1, 9, 7, rot(4, 100.0), 20),
        latent(1, 5, 10, 30, rot(6, 50.0, (2.5, 40, 3.0, 0.5)), 1, 50),
        latent(3, 10, 6, 22, rot(2), None),
        attn(2, 2, 22, 14, rot(0), 34)], loop=(0, 2, 3), eps=1e-3,
        scale=0.25),
    # groups of heads that need more than one tile, wide states
    "wide": config(192, 96, [
        attn(20, 1, 64, 136, rot(64, 1e6), 64),
        latent(20, 64, 80, 128, rot(64, 1e4, (1.0, 128, 32.0, 1.0)), 130, 64),
        light(2, 200, 72, [0.999, 0.6], 64)], scale=1.0),
    # every matrix fits the packed form of the decode path, a loop of all
    "packed": config(128, 96, [
        light(4, 32, 48, [0.99, 0.9, 0.7, 0.2], 160),
        latent(4, 32, 16, 64, rot(32, 1e4, (8.0, 256, 32.0, 1.0)), 33, 128),
        attn(8, 4, 32, 24, rot(16), 64)], loop=(0, 3, 2), scale=3.0),
}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    out = {}
    for name, cfg in MODELS.items():
        d = tmp_path_factory.mktemp(name)
        w = oracle.random_weights(cfg, seed=len(name))
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
    assert rel(got, want) < tol(dtype, 3e-5, 0.04)


# ----------------------------------------------------------------- row steps

@where
@pytest.mark.parametrize("W", [64, 90, 1000, 2100, 9000])
def test_residual_sum(where, W):
    """The plain sum, a vector on top, no base, the embedding row behind;
    rows from far below the eps to large."""
    dev, dt = where
    g = torch.Generator().manual_seed(W)
    eps = 1e-3
    emb = torch.randn(11, W, generator=g).to(dt)
    pre, shift = (1 + 0.3 * torch.randn(W, generator=g) for _ in range(2))
    size = torch.logspace(-3, 1, 9)[:, None]
    x = torch.randn(9, W, generator=g) * size
    y = (torch.randn(9, W, generator=g) * size.flip(0)).to(dt)
    toks = torch.tensor([3, 10, 0, 3, 1, 2, 4, 9, 9], dtype=torch.int32)
    d = lambda t: t.to(dev)
    kw = dict(embed=d(emb), tokens=d(toks))
    f = lambda t: t.to(F64)
    want = f(x) + 0.7 * f(y)
    lim = tol(dt, 1e-6, 4e-3)
    normed = lambda t: oracle.norm(t, f(pre) - 1, eps)
    for yy in [y] + ([y.float()[None] * 0.25 + torch.zeros(4, 1, 1)]
                     if dt == BF16 and dev != "cpu" else []):
        yd = d(yy) if yy.dim() == 2 else ops.Partials(d(yy))
        xo, h = ops.rms_residual(d(x), yd, None, d(pre), 0.7, eps, **kw)
        assert rel(xo, want) < 1e-6 and rel(h, normed(want)) < lim
        xo, h = ops.rms_residual(d(x), yd, None, d(pre), 0.7, eps,
                                 shift=d(shift), **kw)
        assert rel(xo, want + f(shift)) < 1e-6
        assert rel(h, normed(want + f(shift))) < lim
        xo, h = ops.rms_residual(None, yd, None, d(pre), 1.0, eps, bare=True,
                                 shift=d(shift), **kw)
        assert rel(xo, f(y) + f(shift)) < 1e-6
        _, h = ops.rms_residual(d(x), yd, None, None, 0.7, eps, tail=True,
                                need_x=False, **kw)
        assert h.shape == (9, 2 * W) and rel(h[:, :W], want) < lim
        assert torch.equal(h[:, W:].cpu(), emb[toks.long()])
    _, h = ops.rms_residual(None, None, None, None, 1.0, eps, tail=True,
                            need_x=False, **kw)
    assert torch.equal(h[:, :W].cpu(), emb[toks.long()])
    assert torch.equal(h[:, W:].cpu(), emb[toks.long()])


@where
@pytest.mark.parametrize("n,k,rows", [(64, 128, 3), (90, 180, 40),
                                      (96, 640, 80), (32, 64, 1)])
def test_fp32_product(where, n, k, rows):
    """The result is not rounded to the operands' type."""
    dev, dt = where
    g = torch.Generator().manual_seed(n)
    w, x = (torch.randn(m, k, generator=g).to(BF16) for m in (n, rows))
    want = x.to(F64) @ w.to(F64).T
    got = ops.linear_f32(x.to(dev, dt), w.to(dev, dt))
    assert got.dtype == F32 and rel(got, want) < 2e-6
    packed = ops.pack_weight(w.to(dev))
    if dt == BF16 and packed is not None and rows <= 64:
        _, h = ops.rms_residual(x.float().to(dev), None, None, None, 1.0, 0.0,
                                embed=x.to(dev), frag=True)
        got = ops.linear_f32(h, w.to(dev), packed)
        assert rel(got.parts.sum(0), want) < 2e-6


@where
@pytest.mark.parametrize("F,rows", [(64, 1), (192, 33), (200, 5), (1024, 70)])
def test_gated_feed_forward(where, F, rows):
    dev, dt = where
    g = torch.Generator().manual_seed(F)
    K = 128
    w = (torch.randn(2 * F, K, generator=g) / 6).to(BF16)
    x = torch.randn(rows, K, generator=g).to(BF16)
    z = x.to(F64) @ w.to(F64).T
    want = oracle.silu(z[:, :F]) * z[:, F:]
    wd = w.to(dev, dt)
    got = ops.gateup_swiglu(x.to(dev, dt), wd)
    assert rel(got, want) < tol(dt, 2e-6, 8e-3)
    packed = ops.pack_weight_gu(wd)
    if packed is not None and F % 64 == 0 and rows <= 64:
        _, h = ops.rms_residual(x.float().to(dev), None, None, None, 1.0, 0.0,
                                embed=x.to(dev), frag=True)
        act = ops.gateup_swiglu(h, wd, packed)
        eye = torch.eye(F, dtype=BF16, device=dev)
        got = ops.linear(act, eye, packed=ops.pack_weight(eye))
        assert rel(got, want) < 8e-3


# ------------------------------------------------------------------ rotation

ROTS = [rot(8), rot(64, 1e6), rot(2, 10.0), rot(16, 500.0, (4.0, 64, 8.0, 1.0)),
        rot(32, 1e4, (40.0, 4096, 32.0, 1.0)), rot(6, 50.0, (2.5, 40, 3.0, 0.5)),
        rot(24, 1e4, (1.0, 300, 32.0, 1.0)), rot(12, 3.0, (8.0, 7, 20.0, 9.0))]


@pytest.mark.parametrize("r", ROTS, ids=lambda r: "-".join(
    str(v) for v in (r["dims"], *r.get("scaling", {}).values())))
def test_rotation_table(r):
    """Frequencies, the ramp between kept and divided ones, the magnitude,
    at near and far positions."""
    rope = RopeTables(5000, "cpu")(RopeSpec.from_json(r))
    f, mag = oracle.frequencies(r)
    for p in (0, 1, 37, 4999):
        want = torch.tensor([x for fi in f for x in
                             (mag * math.cos(p * fi), mag * math.sin(p * fi))],
                            dtype=F64)
        assert (rope.table[p].to(F64) - want).abs().max() < 1e-6


def test_layers_share_rotation_tables():
    tables = RopeTables(10, "cpu")
    a = tables(RopeSpec(4, 10.0))
    assert tables(RopeSpec(4, 10.0)) is a
    assert tables(RopeSpec(4, 11.0)) is not a


def forms_of(rows, dt, dev, g):
    """A projection as strided rows and, in bf16, as partial sums."""
    n, c = rows.shape
    buf = torch.zeros(n, c + 8 - c % 8, dtype=dt)
    buf[:, :c] = rows
    yield buf.to(dev), buf[:, :c].to(F64)
    if dt == BF16 and dev != "cpu":
        parts = torch.randn(3, *buf.shape, generator=g)
        parts[0, :, :c] += rows
        yield ops.Partials(parts.to(dev)), parts[:, :, :c].to(F64).sum(0)


def two_slots(stores, n, dev, dt):
    """A slot whose pages are not in order, and every pool dirty."""
    cache = HybridCache(stores, n_pages=2 * (n // 16 + 4), max_slots=3,
                        max_ctx=n + 32, device=dev, dtype=dt)
    other, slot = cache.alloc_slot(), cache.alloc_slot()
    cache.ensure(slot, max(1, n // 2))
    cache.ensure(other, 20)
    cache.ensure(slot, n)
    return cache, slot


QKV = [((6, 2, 24, 40), rot(8)), ((3, 1, 9, 7), rot(4)),
       ((4, 4, 64, 136), rot(64, 1e6)), ((2, 1, 32, 16), rot(0)),
       ((40, 8, 128, 128), rot(128, 1e4, (4.0, 64, 8.0, 1.0)))]


@where
@pytest.mark.parametrize("size,r", QKV, ids=lambda v: str(v)[:24])
@pytest.mark.parametrize("n", [1, 70])
def test_split_rotate_append(where, size, r, n):
    """Biases, rotation of the first dimensions only, values as they are;
    nothing else in the pools changes."""
    dev, dt = where
    H, G, D, V = size
    g = torch.Generator().manual_seed(n)
    w = ops.SoftmaxAttn(H, G, D, V, 1.0)
    c = H * D + G * (D + V)
    rows, bias = (torch.randn(k, c, generator=g) for k in (n, 1))
    at, tot = 13, n + 13
    for p, exact_rows in forms_of(rows, dt, dev, g):
        cache, slot = two_slots([RunStore(kv=(G, D, V))], tot, dev, dt)
        rope = RopeTables(cache.max_ctx, dev)(RopeSpec.from_json(r))
        for pool in (cache.key_pool[0], cache.value_pool[0]):
            pool.fill_(3.0)
        sl, pos = rows_of(dev, [slot], [n], [tot])
        q = ops.rope_qkv_append(p, bias[0].to(dev), cache, 0, w, rope, sl,
                                pos)
        wq, wk, wv = (exact_rows + bias.to(F64)).split(
            [H * D, G * D, G * V], 1)
        turn = lambda t, h: oracle.rotate(t.reshape(n, h, D),
                                          range(at, tot), r)
        lim = tol(dt, 1e-6, 4e-3)
        assert rel(q[..., :D], turn(wq, H)) < lim
        assert bool((q[..., D:] == 0).all())
        pages = cache.page_table[slot, :-(-tot // 16)].long()
        kp, vp = (t[0][pages].transpose(1, 2).flatten(0, 1)
                  for t in (cache.key_pool, cache.value_pool))
        assert rel(kp[at:tot, :, :D], turn(wk, G)) < lim
        assert rel(vp[at:tot, :, :V], wv.reshape(n, G, V)) < lim
        for t in (kp, vp):
            assert bool((t[:at] == 3).all()) and bool((t[tot:] == 3).all())
        rest = torch.ones(cache.n_pages + 1, dtype=torch.bool, device=dev)
        rest[pages] = False
        assert bool((cache.key_pool[0][rest] == 3.0).all())
        assert bool((cache.value_pool[0][rest] == 3.0).all())


LATENT = [  # heads, unrotated, rotated, value width, rank
    (4, 32, 16, 40, 88), (1, 5, 6, 10, 30), (20, 64, 64, 48, 128),
    (3, 16, 8, 24, 520), (33, 128, 64, 128, 512), (5, 24, 2, 136, 40)]


def latent_case(dev, dt, size, window=0, seed=0, scale=None):
    H, D, E, V, R = size
    g = torch.Generator().manual_seed(seed)
    uk = (torch.randn(H, D, R, generator=g) / R ** 0.5).to(BF16)
    uv = (torch.randn(H, V, R, generator=g) / R ** 0.5).to(BF16)
    put = lambda t: t.to(dev, dt).contiguous()
    w = ops.LatentWeights(put(uk), put(uk.transpose(1, 2)), put(uv),
                          scale or 1.4 * (D + E) ** -0.5, E, window)
    store = RunStore(latent=-(-(R + E) // 8) * 8)
    return g, uk.to(F64), uv.to(F64), w, store


@where
@pytest.mark.parametrize("size", LATENT, ids=str)
@pytest.mark.parametrize("n", [1, 70])
def test_latent_split_rotate_append(where, size, n):
    """Only the rotated part of a head turns, only the latent is normed."""
    dev, dt = where
    H, D, E, V, R = size
    g, _, _, w, store = latent_case(dev, dt, size)
    r = rot(E, 300.0, (3.0, 50, 6.0, 1.0))
    nw = 1 + 0.3 * torch.randn(R, generator=g)
    rows = torch.randn(n, H * (D + E) + R + E, generator=g)
    at, tot, eps = 13, n + 13, 0.3
    for p, exact_rows in forms_of(rows, dt, dev, g):
        cache, slot = two_slots([store], tot, dev, dt)
        rope = RopeTables(cache.max_ctx, dev)(RopeSpec.from_json(r))
        sl, pos = rows_of(dev, [slot], [n], [tot])
        q = ops.latent_rope_append(p, cache, 0, w, nw.to(dev), eps, rope, sl,
                                   pos)
        wq, c, k = exact_rows.split([H * (D + E), R, E], 1)
        wq = wq.reshape(n, H, D + E)
        lim = tol(dt, 1e-6, 4e-3)
        turn = lambda t: oracle.rotate(t, range(at, tot), r)
        want = torch.cat([wq[..., :D], turn(wq[..., D:])], -1)
        assert rel(q.view(n, H, D + E), want) < lim
        pages = cache.page_table[slot, :-(-tot // 16)].long()
        row = cache.latent_pool[0][pages].flatten(0, 1)
        assert rel(row[at:tot, :R],
                   oracle.rms(c, eps) * nw.to(F64)) < lim
        assert rel(row[at:tot, R:R + E], turn(k)) < lim
        assert bool((row[:at] == 0).all()) and bool((row[tot:] == 0).all())
        assert bool((row[:, R + E:] == 0).all())


# --------------------------------------------------------- softmax attention

def soft(H, G, D, V, window=0, sink=None, seed=0, scale=None, dev="cpu"):
    g = torch.Generator().manual_seed(seed)
    s = None if sink is None else sink + torch.randn(H, generator=g)
    return g, ops.SoftmaxAttn(H, G, D, V, scale or 1.5 * D ** -0.5,
                              None if s is None else s.to(dev), window)


def new_cache(dev, dt, w, kv):
    return HybridCache([RunStore(kv=(w.kv_heads, w.dim, w.vdim))],
                       n_pages=3 * (kv // 16 + 2), max_slots=3,
                       max_ctx=kv + 16, device=dev, dtype=dt)


def put_kv(cache, w, slot, at, q, k, v):
    """Append rows through the op, without rotation and bias."""
    dev, dt = cache.key_pool[0].device, cache.key_pool[0].dtype
    n = q.shape[0]
    cache.ensure(slot, at + n)
    sl, pos = rows_of(dev, [slot], [n], [at + n])
    p = torch.cat([t.reshape(n, -1) for t in (q, k, v)], 1).to(dev, dt)
    still = RopeTables(cache.max_ctx, dev)(RopeSpec(0, 1.0))
    return ops.rope_qkv_append(p, None, cache, 0, w, still, sl, pos), sl, \
        pos, meta_for(dev, [slot], [n], [at + n])


def o_attention(w, q, k, v, start=0, window=None, sink=True):
    """q [T, H, D], k [N, G, D], v [N, G, V] -> [T, H*V]"""
    f = lambda t: t.to("cpu", F64)
    R = w.heads // w.kv_heads
    return torch.cat([oracle.softmax_attention(
        f(q)[:, h], f(k)[:, h // R], f(v)[:, h // R], w.scale,
        window or w.window or None,
        f(w.sink)[h] if sink and w.sink is not None else None, start)
        for h in range(w.heads)], -1)


@where
@pytest.mark.parametrize("size", [(6, 2, 24, 40), (3, 1, 9, 7),
                                  (20, 1, 64, 136), (4, 4, 80, 64),
                                  (8, 2, 128, 128), (2, 1, 256, 250)],
                         ids=str)
@pytest.mark.parametrize("window,sink", [(0, 1.0), (0, None), (1, 0.0),
                                         (48, 2.0), (100, None)])
@pytest.mark.parametrize("form", ["whole", "large tiles", "portions",
                                  "single"])
def test_softmax_attention(where, size, window, sink, form, monkeypatch):
    """Whole prompts, portions down to two tokens and single tokens over a
    context whose length is no multiple of anything, with pages handed out
    in a mixed order."""
    dev, dt = where
    if form == "large tiles":
        if dev == "cpu":
            pytest.skip("the CPU form has no tiles")
        from ollamamq_amd.ops import hip
        monkeypatch.setattr(hip, "ATTN_LARGE", 0)
    H, G, D, V = size
    kv = 130 if form == "single" else 260
    g, w = soft(H, G, D, V, window, sink, seed=window, dev=dev)
    q, k = (torch.randn(kv, h, D, generator=g).to(dt) for h in (H, G))
    v = torch.randn(kv, G, V, generator=g).to(dt)
    cache = new_cache(dev, dt, w, kv)
    other, slot = cache.alloc_slot(), cache.alloc_slot()
    lens = {"whole": [kv], "large tiles": [kv], "single": [1] * kv,
            "portions": [90, 2, 2, 31, 1, 64, 8, 9, 53]}[form]
    got, at = [], 0
    for n in lens:
        cache.ensure(other, min(kv, 40 + at))
        qq, sl, pos, meta = put_kv(cache, w, slot, at, q[at:at + n],
                                   k[at:at + n], v[at:at + n])
        got.append(ops.softmax_attention(qq, cache, 0, w, sl, pos,
                                         meta).cpu())
        at += n
    want = o_attention(w, q, k, v)
    assert rel(torch.cat(got), want) < tol(dt, 3e-6, 1.2e-2)


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
    G, D, V = w.kv_heads, w.dim, w.vdim
    rest = torch.zeros(k.shape[0], w.heads, D)
    put_kv(cache, w, slot, 0, rest, k, v)
    qq = torch.zeros(n, w.heads, cache.key_pool[0].shape[3], dtype=dt)
    qq[..., :D] = q1
    sl, pos = rows_of(dev, [slot], [n], [first + n])
    return ops.softmax_attention(qq.to(dev), cache, 0, w, sl, pos, meta_for(
        dev, [slot], [n], [first + n])).cpu()


@where
@pytest.mark.parametrize("window", [1, 2, 15, 16, 17, 33, 64, 65, 200])
@pytest.mark.parametrize("n", [1, 2, 40])
def test_softmax_window_edges(where, window, n):
    """The last key inside and the first key outside each window: one token
    more or less shows, in decoding and in portions."""
    dev, dt = where
    H, G, D, V, kv = 4, 2, 32, 24, 290
    g, w = soft(H, G, D, V, window, 4.0, seed=3, scale=1.0, dev=dev)
    for first in (window - 1, 63, 64, 79, 200, kv - n):
        if not 0 <= first <= kv - n:
            continue
        for edge in sorted({first, first + n - 1}):
            inside, outside = edge - window + 1, edge - window
            marks = [j for j in (inside, outside) if j >= 0]
            q1, k = aimed(w, g, kv, marks, dt)
            v = torch.randn(kv, G, V, generator=g).to(dt)
            got = run_at(dev, dt, w, q1, k, v, first, n)
            row = edge - first
            want = o_attention(w, q1.expand(n, H, D), k, v, first)
            assert rel(got, want) < tol(dt, 1e-5, 2e-2), (first, edge)
            for off in ((1,) if outside >= 0 else ()) + \
                    ((-1,) if window > 1 and inside >= 0 else ()):
                other = o_attention(w, q1[None], k, v, edge, window + off)
                assert rel(other[0], want[row]) > 0.3, "the edge must show"


@where
@pytest.mark.parametrize("n", [1, 2, 40, 300])
def test_far_keys_are_found(where, n):
    """One loud key among hundreds: first tokens, page, chunk and tile
    borders, the query's own token."""
    dev, dt = where
    H, G, D, V, kv = 2, 1, 32, 24, 700
    g, w = soft(H, G, D, V, 0, 1.0, seed=5, scale=1.0, dev=dev)
    for j in (0, 1, 15, 16, 31, 32, 63, 64, 65, 127, 128, 255, 256, 399,
              kv - n):
        q1, k = aimed(w, g, kv, [j], dt)
        v = torch.randn(kv, G, V, generator=g).to(dt)
        got = run_at(dev, dt, w, q1, k, v, kv - n, n)
        want = o_attention(w, q1.expand(n, H, D), k, v, kv - n)
        cos = torch.cosine_similarity(want[-1, :V], v[j, 0].to(F64), 0)
        assert cos > 0.9, "the aimed key must stand out"
        assert rel(got, want) < tol(dt, 1e-5, 2e-2), j


@where
@pytest.mark.parametrize("level", [-60.0, 0.0, 30.0, 200.0])
@pytest.mark.parametrize("n", [1, 40])
def test_sink(where, level, n):
    """Sinks from far below all scores to far above, per head; scores far
    from zero."""
    dev, dt = where
    H, G, D, V, kv = 4, 2, 32, 24, 90
    g, w = soft(H, G, D, V, 0, level, seed=9, scale=2.0, dev=dev)
    q1, k = aimed(w, g, kv, [7], dt)             # one score of 32
    v = torch.randn(kv, G, V, generator=g).to(dt)
    want = o_attention(w, q1.expand(n, H, D), k, v, kv - n)
    got = run_at(dev, dt, w, q1, k, v, kv - n, n)
    bare = o_attention(w, q1.expand(n, H, D), k, v, kv - n, sink=False)
    if level == 30.0:
        assert rel(want, bare) > 0.02
    if level == 200.0:
        assert want.abs().max() < 1e-6
        assert got.abs().max() < 1e-6
    else:
        assert rel(got, want) < tol(dt, 1e-5, 2e-2)
    low = run_at(dev, dt, w._replace(scale=-2.0), q1, k, v, kv - n, n)
    want = o_attention(w._replace(scale=-2.0), q1.expand(n, H, D), k, v,
                       kv - n)
    assert (low.to(F64) - want).abs().max() < tol(dt, 1e-5, 2e-2)


# ---------------------------------------------------------- latent attention

def o_latent(uk, uv, q, row, w, start=0, window=None):
    R, E = uk.shape[2], w.rot_dim
    f = lambda t: t.to("cpu", F64)
    return oracle.latent_heads(f(q), f(row)[:, :R], f(row)[:, R:R + E], uk,
                               uv, w.scale, window or w.window or None,
                               start)


def fill_rows(cache, slot, row):
    n = row.shape[0]
    cache.ensure(slot, n)
    pages = cache.page_table[slot, :-(-n // 16)].long()
    pool = cache.latent_pool[0]
    full = torch.zeros(len(pages) * 16, pool.shape[2], dtype=row.dtype)
    full[:n, :row.shape[1]] = row
    pool[pages] = full.view(-1, 16, pool.shape[2]).to(pool.device)


@where
@pytest.mark.parametrize("size", LATENT, ids=str)
@pytest.mark.parametrize("window", [0, 1, 48, 130])
@pytest.mark.parametrize("form", ["whole", "portions", "single"])
def test_latent_attention(where, size, window, form):
    """Whole prompts, portions and single tokens; absorbed and expanded
    forms, rotated part and gate."""
    dev, dt = where
    H, D, E, V, R = size
    kv = 110 if form == "single" else 270
    g, uk, uv, w, store = latent_case(dev, dt, size, window, 3)
    q = torch.randn(kv, H, D + E, generator=g).to(dt)
    row = torch.randn(kv, R + E, generator=g).to(dt)
    gate = torch.randn(kv, H * V + 8, generator=g).to(dt)
    cache = HybridCache([store], n_pages=3 * (kv // 16 + 2), max_slots=3,
                        max_ctx=kv + 16, device=dev, dtype=dt)
    other, slot = cache.alloc_slot(), cache.alloc_slot()
    cache.ensure(slot, 50)
    cache.ensure(other, 40)
    fill_rows(cache, slot, row)
    lens = {"whole": [kv], "single": [1] * kv,
            "portions": [90, 2, 2, 31, 1, 64, 17, 9, 54]}[form]
    got, at = [], 0
    for n in lens:
        sl, pos = rows_of(dev, [slot], [n], [at + n])
        meta = meta_for(dev, [slot], [n], [at + n])
        gp = gate[at:at + n].to(dev)
        if n <= 2 and dt == BF16 and dev != "cpu":
            gp = ops.Partials(torch.stack([gp.float() - 1, gp * 0 + 1.0]))
        got.append(ops.latent_attention(
            q[at:at + n].flatten(1).to(dev), cache, 0, w, sl, pos, meta,
            gate=ops.Columns(gp, 8)).cpu())
        at += n
    want = o_latent(uk, uv, q, row, w) * oracle.sigmoid(
        gate[:, 8:].to(F64))
    assert rel(torch.cat(got), want) < tol(dt, 5e-6, 2e-2)


def aimed_rows(g, H, D, E, R, uk, kv, marks, by):
    """Rows at `marks` stand out for one query of every head, by the latent
    or by the rotated part."""
    row = 0.05 * torch.randn(kv, R + E, generator=g, dtype=F64)
    q = torch.zeros(H, D + E, dtype=F64)
    if by == "rotated":
        d = torch.randn(E, generator=g, dtype=F64)
        d /= d.norm()
        q[:, D:] = 4 * d
        for j in marks:
            row[j, R:] = 4 * d
            row[j, :R] = torch.randn(R, generator=g, dtype=F64)
    else:
        c = torch.randn(R, generator=g, dtype=F64)
        q[:, :D] = uk @ c
        q[:, :D] *= 4 / q[:, :D].norm(dim=-1, keepdim=True)
        reach = torch.stack([(uk[h] @ c) @ q[h, :D] for h in range(H)]).min()
        # values of their own, from directions that no query sees
        seen = torch.linalg.qr(torch.stack(
            [uk[h].T @ q[h, :D] for h in range(H)], 1)).Q
        for j in marks:
            own = 3 * torch.randn(R, generator=g, dtype=F64)
            row[j, :R] = c * 10 / reach + own - seen @ (seen.T @ own)
    return q, row


@where
@pytest.mark.parametrize("by", ["latent", "rotated"])
@pytest.mark.parametrize("window", [1, 2, 16, 17, 33, 64, 65, 200])
@pytest.mark.parametrize("n", [1, 2, 40])
def test_latent_window_edges(where, window, n, by):
    dev, dt = where
    size = H, D, E, V, R = 3, 32, 16, 24, 40
    kv = 290
    g, uk, uv, w, store = latent_case(dev, dt, size, window, 7, scale=1.0)
    for first in (window - 1, 63, 64, 79, 200, kv - n):
        if not 0 <= first <= kv - n:
            continue
        for edge in sorted({first, first + n - 1}):
            inside, outside = edge - window + 1, edge - window
            marks = [j for j in (inside, outside) if j >= 0]
            q, row = aimed_rows(g, H, D, E, R, uk, kv, marks, by)
            q, row = q.to(dt), row.to(dt)
            cache = HybridCache([store], n_pages=40, max_slots=2,
                                max_ctx=kv + 16, device=dev, dtype=dt)
            slot = cache.alloc_slot()
            fill_rows(cache, slot, row)
            sl, pos = rows_of(dev, [slot], [n], [first + n])
            got = ops.latent_attention(
                q.flatten().expand(n, -1).contiguous().to(dev), cache, 0, w,
                sl, pos, meta_for(dev, [slot], [n], [first + n])).cpu()
            want = o_latent(uk, uv, q.expand(n, -1, -1), row, w, first)
            # expanded keys are bf16, and most of each is outside the score
            assert rel(got, want) < tol(dt, 1e-5, 6e-2), (first, edge)
            for off in ((1,) if outside >= 0 else ()) + \
                    ((-1,) if window > 1 and inside >= 0 else ()):
                other = o_latent(uk, uv, q[None], row, w, edge, window + off)
                assert rel(other[0], want[edge - first]) > 0.2, \
                    "the edge must show"


@where
@pytest.mark.parametrize("by", ["latent", "rotated"])
@pytest.mark.parametrize("n", [1, 2, 40, 300])
def test_latent_far_keys(where, n, by):
    dev, dt = where
    size = H, D, E, V, R = 2, 32, 16, 24, 64
    kv = 700
    g, uk, uv, w, store = latent_case(dev, dt, size, 0, 8, scale=1.0)
    for j in (0, 1, 15, 16, 63, 64, 65, 255, 256, 399, kv - n):
        q, row = aimed_rows(g, H, D, E, R, uk, kv, [j], by)
        q, row = q.to(dt), row.to(dt)
        cache = HybridCache([store], n_pages=60, max_slots=2,
                            max_ctx=kv + 16, device=dev, dtype=dt)
        slot = cache.alloc_slot()
        fill_rows(cache, slot, row)
        sl, pos = rows_of(dev, [slot], [n], [kv])
        got = ops.latent_attention(
            q.flatten().expand(n, -1).contiguous().to(dev), cache, 0, w, sl,
            pos, meta_for(dev, [slot], [n], [kv])).cpu()
        want = o_latent(uk, uv, q.expand(n, -1, -1), row, w, kv - n)
        cos = torch.cosine_similarity(want[-1, :V],
                                      uv[0] @ row[j, :R].to(F64), 0)
        assert cos > 0.9, "the aimed key must stand out"
        assert rel(got, want) < tol(dt, 1e-5, 3e-2), j


# ------------------------------------------------------- lightning attention

def lightning_case(dev, dt, H, D, V, decay, n, seed=0):
    g = torch.Generator().manual_seed(seed)
    norm = 1 + 0.3 * torch.randn(H * V, generator=g)
    steps = torch.arange(ops.LIGHTNING_CHUNK + 1, dtype=F64)
    powers = (torch.tensor(decay, dtype=F64)[:, None] ** steps).float()
    w = ops.LightningWeights(
        H, D, V, (0, H * D, 2 * H * D, 2 * H * D + H * V), powers.to(dev),
        norm.to(dev), 1e-4)
    p = torch.randn(n, 2 * H * (D + V), generator=g)
    # heads of unequal magnitude keep their proportions in the norm
    p[:, 2 * H * D:2 * H * D + V] *= 5
    return g, w, p.to(dt)


def o_lightning(w, p, decay):
    H, D, V = w.heads, w.dim, w.vdim
    q, k, v, gate = p.to(F64).split([H * D, H * D, H * V, H * V], 1)
    n = p.shape[0]
    o, S = oracle.lightning_heads(
        oracle.silu(q).view(n, H, D), oracle.silu(k).view(n, H, D),
        oracle.silu(v).view(n, H, V), decay)
    return oracle.gated_norm(o.reshape(n, H * V), w.norm.to("cpu", F64),
                             gate, w.eps), S


SIZES = [(3, 24, 40), (2, 9, 7), (4, 64, 64), (2, 128, 128), (1, 200, 136),
         (1, 300, 16), (2, 16, 300)]
DECAYS = [0.999, 0.3, 0.9, 0.0]


@where
@pytest.mark.parametrize("size", SIZES, ids=str)
@pytest.mark.parametrize("form", ["whole", "portions", "single"])
def test_lightning(where, size, form):
    """A dirty slot is taken as empty at position 0 and carried after that;
    chunks, token by token and portions of both agree."""
    dev, dt = where
    H, D, V = size
    decay = DECAYS[:H]
    n = 75 if form == "single" else 210
    g, w, p = lightning_case(dev, dt, H, D, V, decay, n)
    state = torch.full((3, H, D, V), 7.0, device=dev)
    lens = {"whole": [n], "single": [1] * n,
            "portions": [70, 2, 3, 1, 64, 5, 65]}[form]
    got, at = [], 0
    for m in lens:
        sl, pos = rows_of(dev, [1], [m], [at + m])
        pd = p[at:at + m].to(dev)
        if m < 3 and dt == BF16 and dev != "cpu":
            pd = ops.Partials(torch.stack([pd.float() - 1, pd * 0 + 1.0]))
        got.append(ops.lightning(pd, w, state, sl, pos, meta_for(
            dev, [1], [m], [at + m])).cpu())
        at += m
    want, S = o_lightning(w, p, decay)
    assert rel(torch.cat(got), want) < tol(dt, 5e-6, 1e-2)
    assert rel(state[1], S) < tol(dt, 5e-6, 5e-3)
    assert bool((state[0] == 7).all()) and bool((state[2] == 7).all())


@where
@pytest.mark.parametrize("n", [1, 2, 63, 64, 65, 150])
def test_lightning_remembers_far_tokens(where, n):
    """One loud token long ago is what a slow head returns, at chunk borders
    and from before the portion; a fast head has forgotten it."""
    dev, dt = where
    H, D, V, kv = 2, 32, 24, 400
    decay = [1.0, 0.5]
    g, w, p = lightning_case(dev, dt, H, D, V, decay, kv)
    p = 0.02 * p
    for j in (0, 63, 64, 128, 200, kv - n):
        x = p.clone()
        x[j, H * D:2 * H * D + H * V] = 4 + torch.randn(
            H * (D + V), generator=g).to(dt)
        x[-1, :H * D] = 2.0
        state = torch.full((2, H, D, V), -3.0, device=dev)
        got = []
        for at, m in ((0, kv - n), (kv - n, n)):
            sl, pos = rows_of(dev, [0], [m], [at + m])
            got.append(ops.lightning(
                x[at:at + m].to(dev), w, state, sl, pos,
                meta_for(dev, [0], [m], [at + m])).cpu())
        want, _ = o_lightning(w, x, decay)
        assert rel(got[1][-1:], want[-1:]) < tol(dt, 1e-5, 1e-2), j


@where
def test_lightning_batch(where):
    """Single tokens, short and long portions of several slots in one
    call."""
    dev, dt = where
    H, D, V, decay = 2, 24, 40, [0.98, 0.7]
    lens, before = [1, 1, 3, 70, 130], [40, 0, 5, 64, 0]
    cases = [lightning_case(dev, dt, H, D, V, decay, b + n, i)
             for i, (n, b) in enumerate(zip(lens, before))]
    w = cases[0][1]
    state = torch.full((6, H, D, V), 9.0, device=dev)
    slots = [3, 0, 5, 1, 2]
    for s, (_, _, p), b in zip(slots, cases, before):
        if b:
            sl, pos = rows_of(dev, [s], [b], [b])
            ops.lightning(p[:b].to(dev), w, state, sl, pos,
                          meta_for(dev, [s], [b], [b]))
    tot = [b + n for b, n in zip(before, lens)]
    sl, pos = rows_of(dev, slots, lens, tot)
    got = ops.lightning(
        torch.cat([p[b:] for (_, _, p), b in zip(cases, before)]).to(dev), w,
        state, sl, pos, meta_for(dev, slots, lens, tot, n_decode=2)).cpu()
    for (_, _, p), b, part in zip(cases, before, got.split(lens)):
        assert rel(part, o_lightning(w, p, decay)[0][b:]) \
            < tol(dt, 5e-6, 1e-2)


# --------------------------------------------------------------- whole models

def test_config_reaches_every_constant(models):
    kc = KavedraConfig.from_json(models["mixed"][1])
    assert (kc.eps, kc.logit_scale, kc.loop) == (1e-5, 1.5, (1, 4, 2))
    assert kc.runs == [(0, None), (1, 0), (2, None), (3, None), (1, 1),
                       (2, None), (3, None), (4, None)]
    a, b, c, d, e = kc.layers
    assert a.decay == (0.3, 0.9, 0.995) and a.ff == 80
    assert (b.kv_rank, b.rot_dim, b.window, b.row) == (56, 8, 37, 64)
    assert b.rope == RopeSpec(8, 500.0, (4.0, 64.0, 8.0, 1.0))
    assert (c.heads, c.kv_heads, c.dim, c.vdim, c.ff) == (6, 2, 24, 40, None)
    stores = kc.run_stores()
    assert len(stores) == 8
    assert stores[2].kv == (2, 24, 40) and stores[5].kv == (2, 24, 40)
    assert stores[1].latent == 64 and stores[7].latent == 48
    assert KavedraConfig.from_json(
        dict(models["mixed"][1], loop={"start": 2, "stop": 2, "times": 3})
    ).runs == [(i, None) for i in range(5)]


@exact
@pytest.mark.parametrize("name", list(MODELS))
def test_every_layer(models, where, name):
    """The residual stream after every layer run."""
    dev, dt = where
    path, cfg, w = models[name]
    toks = tokens_for(name, 40)
    _, want = oracle.run(cfg, w, toks)
    kc = config_from_folder(path)
    model = build_model(kc, device=dev, dtype=dt)
    kv = cache_for_model(kc, n_pages=8, max_slots=2, max_ctx=64, device=dev,
                         dtype=dt)
    slot = kv.alloc_slot()
    kv.ensure(slot, 40)
    sl, pos = rows_of(dev, [slot], [40], [40])
    out = []
    model.forward(torch.tensor(toks, dtype=torch.int32, device=dev), pos, kv,
                  sl, meta_for(dev, [slot], [40], [40]), layer_out=out)
    assert len(out) == len(want) == len(kc.runs)
    for got, ref in zip(out, want):
        assert got.dtype == F32 and rel(got, ref) < 1e-5


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
    """Every window passes over decoded tokens several times."""
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
    kc = config_from_folder(path)
    kv = cache_for_model(kc, n_pages=40, max_slots=3, max_ctx=160,
                         device=dev, dtype=dt)
    eng = LlamaEngine(build_model(kc, device=dev, dtype=dt), kv, max_batch=3,
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
    kc = config_from_folder(path)

    def run(graphs):
        kv = cache_for_model(kc, n_pages=64, max_slots=6, max_ctx=160,
                             device="cuda:0", dtype=dt)
        eng = LlamaEngine(build_model(kc, device="cuda:0", dtype=dt), kv,
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
    kc = config_from_folder(path)
    kv = cache_for_model(kc, n_pages=users * 4, max_slots=users, max_ctx=64,
                         device="cuda:0", dtype=BF16)
    eng = LlamaEngine(build_model(kc, device="cuda:0", dtype=BF16), kv,
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
    cfg = PRESETS["kavedra-tiny"]
    kv = cache_for_model(cfg, n_pages=32, max_slots=2, max_ctx=128,
                         device=dev, dtype=dt)
    model = build_model(cfg, device=dev, dtype=dt, seed=3)
    assert model.weight_bytes() > 0 and cfg.weight_bytes() > 0
    eng = LlamaEngine(model, kv, max_batch=2)
    out = generate(eng, [[1, 2, 3], [4] * 20], 5)
    assert all(len(o) == 5 for o in out)
    h = torch.tensor(eng.embed([1, 2, 3]), dtype=F64)
    assert len(h) == cfg.width
    # the logits' scale stays out of the embedding
    gain = model.final_norm.cpu().to(F64)
    assert abs((h / gain).pow(2).mean() - 1) < 0.05
    assert cfg.model_info()["block_runs"] == 6


# ------------------------------------------------------------ loading, runner

def test_bad_checkpoints_are_refused(models, tmp_path):
    path, cfg, w = models["odd"]
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    bad = dict(w)
    bad["l1.mix.k.b"] = torch.zeros(3, dtype=BF16)
    save_file(bad, str(tmp_path / "model.safetensors"))
    with pytest.raises(ValueError, match="l1.mix.k.b"):
        build_model(config_from_folder(str(tmp_path)))
    del bad["l1.mix.k.b"]
    save_file(bad, str(tmp_path / "model.safetensors"))
    with pytest.raises(KeyError, match="l1.mix.k.b"):
        build_model(config_from_folder(str(tmp_path)))

    def changed(i, mixer=None, **kw):
        other = json.loads(json.dumps(cfg))
        other["layers"][i].update(kw)
        other["layers"][i]["mixer"].update(mixer or {})
        return KavedraConfig.from_json(other)

    with pytest.raises(ValueError, match="something"):
        changed(0, type="something")
    with pytest.raises(ValueError, match="moe"):
        changed(0, mlp={"kind": "moe", "ff": 3})
    with pytest.raises(ValueError, match="2 decays"):
        changed(0, {"decay": [0.5, 0.5]})
    with pytest.raises(ValueError, match="evenly"):
        changed(1, {"kv_heads": 2})
    with pytest.raises(ValueError, match="10 rotated"):
        changed(1, {"rot": rot(10)})
    with pytest.raises(ValueError, match="rot_dim"):
        changed(2, {"rot_dim": 4})
    with pytest.raises(ValueError, match="3 rotated"):
        changed(1, {"rot": rot(3)})
    with pytest.raises(ValueError, match="window"):
        changed(2, {"mask": {"size": 0}})
    with pytest.raises(ValueError, match="does not fit"):
        KavedraConfig.from_json(dict(cfg, loop={"start": 2, "stop": 9,
                                                "times": 1}))
    with pytest.raises(ValueError, match="parallel"):
        build_model(KavedraConfig.from_json(cfg), tp_size=2)


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
    register_checkpoint(f"kavedra-folder={models['mixed'][0]}")
    try:
        w = Worker(0, max_batch=2, default_ctx=128)
        assert "kavedra-folder" in w.available_models()
        q = queue.Queue()
        w.generate("kavedra-folder", [1, 2, 3], GenParams(max_tokens=6),
                   lambda t, done: q.put((t, done)))
        out = []
        while True:
            t, done = q.get(timeout=60)
            if done:
                break
            out.append(t)
        assert len(out) == 6
        assert w.unload("kavedra-folder") is None
    finally:
        PRESETS.pop("kavedra-folder")
