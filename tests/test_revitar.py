"""The Revitar design against a plain float64 statement of its equations
(revitar_oracle.py): every mechanism alone, then whole models fed in
portions, in batches and through reused memory, then generation.

The same tests run on the CPU and, in fp32 and bf16, on the GPU kernels.
"""
import json
import os
import subprocess

import pytest
import torch
from safetensors.torch import save_file

import revitar_oracle as oracle
from hybrid_common import (BF16, F32, F64, GPU, cut, exact, generate,
                           meta_for, rel, rows_of, run_portions, tol, where)
from ollamamq_amd.engine import (GenParams, HybridCache, LlamaEngine,
                                 cache_for_model)
from ollamamq_amd.engine.kvcache import RunStore
from ollamamq_amd.engine.trace import make_engine
from ollamamq_amd.models import (RevitarConfig, build_model,
                                 config_from_folder)
from ollamamq_amd.ops import interface as ops

REPO = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def layer(heads, kv_heads, dim, vdim, window, moe=None, scale=None,
          softcap=15.0):
    """moe: (experts, top, ff)"""
    return {"type": "attention",
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                      "vdim": vdim, "scale": scale or 1.7 * dim ** -0.5,
                      "softcap": softcap, "mask": {"size": window}},
            "mlp": {"kind": "moe", "expert": {"ff": moe[2]},
                    "router": {"experts": moe[0], "top": moe[1]}}
            if moe else None}


def config(width, vocab, layers, eps=1e-5, scale=0.6, mult=0.4):
    return {"architecture": "Revitar", "width": width, "vocab": vocab,
            "layers": layers, "norm": {"eps": eps},
            "embedding": {"scale": scale}, "residual_mult": mult}


MODELS = {
    # no two layers alike; value heads wider and narrower than key heads,
    # shared and single key heads, one layer without a feed-forward
    "mixed": config(128, 200, [
        layer(6, 2, 24, 40, 37, (5, 2, 80)),
        layer(4, 4, 48, 16, 500),
        layer(8, 1, 16, 72, 64, (3, 1, 48), softcap=2.0)]),
    # sizes that fit no tile, a window of one token, every expert chosen
    "odd": config(90, 131, [
        layer(3, 1, 9, 7, 5, (2, 2, 34)),
        layer(5, 5, 18, 10, 1000, (7, 3, 20)),
        layer(1, 1, 22, 14, 1, (1, 1, 50))], eps=1e-3, scale=1.0, mult=1.0),
    # groups of heads that need more than one tile, more experts than lanes
    # of a tile
    "wide": config(192, 96, [
        layer(20, 1, 64, 136, 130, (19, 4, 64)),
        layer(4, 2, 256, 64, 17, (4, 2, 200))], scale=2.5),
    # every matrix fits the packed form of the decode path
    "packed": config(128, 96, [
        layer(4, 2, 40, 48, 33, (6, 3, 128)),
        layer(2, 1, 32, 32, 100, (9, 2, 64)),
        layer(4, 4, 8, 16, 16)], mult=0.7),
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
    key = (name, tuple(tokens))
    if key not in _ORACLE:
        _, cfg, w = models[name]
        _ORACLE[key] = oracle.run(cfg, w, tokens)[0]
    return _ORACLE[key]


def tokens_for(name, n, seed=0):
    g = torch.Generator().manual_seed(seed * 1000 + n)
    return torch.randint(0, MODELS[name]["vocab"], (n,), generator=g).tolist()


def check(got, want, dtype):
    """In bf16 a token whose router has a close call may go to another
    expert, so a few rows may differ; in fp32 none."""
    if dtype == F32:
        assert rel(got, want) < 3e-5
        return
    err = (got.to("cpu", F64) - want).pow(2).mean(-1).sqrt() \
        / want.pow(2).mean().sqrt()
    err = err.sort().values
    assert err[int(0.9 * (len(err) - 1))] < 0.05, err
    assert torch.isfinite(err).all()


# ---------------------------------------------------------------- mechanisms

@where
@pytest.mark.parametrize("W", [64, 90, 1000, 2100, 9000])
def test_rms_residual(where, W):
    """Rows from far below the eps to large; post norm, scaled sum, pre
    norm, row selection, scaled embedding."""
    dev, dt = where
    g = torch.Generator().manual_seed(W)
    eps, mult = 1e-3, 0.37
    emb = torch.randn(11, W, generator=g).to(dt)
    post, pre = (1 + 0.3 * torch.randn(W, generator=g) for _ in range(2))
    size = torch.logspace(-3, 1, 9)[:, None]
    x = torch.randn(9, W, generator=g) * size
    y = (torch.randn(9, W, generator=g) * size.flip(0)).to(dt)
    d = lambda t: t.to(dev)
    e = d(emb)
    want = x.to(F64) + mult * oracle.rms_norm(y.to(F64), post.to(F64), eps)
    xo, h = ops.rms_residual(d(x), d(y), d(post), None, mult, eps, embed=e)
    assert rel(xo, want) < 1e-6
    assert h.dtype == dt and rel(h, want) < tol(dt, 1e-6, 4e-3)
    _, h = ops.rms_residual(d(x), d(y), d(post), d(pre), mult, eps, embed=e,
                            rows=torch.tensor([7, 2, 2], device=dev),
                            need_x=False)
    assert rel(h, oracle.rms_norm(want, pre.to(F64), eps)[[7, 2, 2]]) \
        < tol(dt, 1e-6, 4e-3)
    toks = torch.tensor([3, 10, 0, 3], dtype=torch.int32)
    xo, h = ops.rms_residual(None, None, None, None, mult, eps, embed=e,
                             tokens=d(toks), embed_scale=0.25)
    assert rel(xo, emb[toks.long()].to(F64) * 0.25) < 1e-6
    # a token's rows with their shares
    parts = torch.randn(9, 3, W, generator=g).to(dt)
    share = torch.rand(9, 3, generator=g)
    want = x.to(F64) + mult * oracle.rms_norm(
        (parts.to(F64) * share.to(F64)[..., None]).sum(1), post.to(F64), eps)
    for p in {dt: parts, F32: parts.float()}.values():
        xo, _ = ops.rms_residual(d(x), ops.Weighted(d(p), d(share)), d(post),
                                 None, mult, eps, embed=e)
        assert rel(xo, want) < 1e-6
    if dev != "cpu" and dt == BF16:
        split = torch.randn(4, 9, W, generator=g)
        want = x.to(F64) + mult * oracle.rms_norm(
            split.to(F64).sum(0), post.to(F64), eps)
        xo, _ = ops.rms_residual(d(x), ops.Partials(d(split)), d(post), None,
                                 mult, eps, embed=e)
        assert rel(xo, want) < 1e-6


def attn_params(dev, H, G, D, V, window, seed=0, scale=None, softcap=15.0,
                bias=-1.0):
    g = torch.Generator().manual_seed(seed)
    decay = 0.5 + 0.5 * torch.rand(H, generator=g)
    reach = 0.02 + torch.rand(H, generator=g)
    b = bias + 0.5 * torch.randn(H, generator=g)
    w = ops.SigmoidAttn(H, G, D, V, scale or 1.5 * D ** -0.5, softcap,
                        decay.to(dev), reach.to(dev), b.to(dev), window)
    return g, w


def new_cache(dev, dt, w, kv, slots=3, pages=None):
    return HybridCache([RunStore(kv=(w.kv_heads, w.dim, w.vdim))],
                       n_pages=pages or 3 * (kv // 16 + 2), max_slots=slots,
                       max_ctx=kv + 16, device=dev, dtype=dt)


def put_kv(cache, w, slot, at, q, k, v):
    """Append rows through the op, the norms without weights and eps."""
    dev, dt = cache.key_pool[0].device, cache.key_pool[0].dtype
    n = q.shape[0]
    cache.ensure(slot, at + n)
    sl, pos = rows_of(dev, [slot], [n], [at + n])
    p = torch.cat([t.reshape(n, -1) for t in (q, k, v)], 1).to(dev, dt)
    one = lambda t: torch.ones(t[0].numel(), device=dev)
    return ops.qk_norm_append(p, cache, 0, w, one(q), one(k), 0.0, sl, pos), \
        sl, pos, meta_for(dev, [slot], [n], [at + n])


def unit(t):
    """Rows with mean square one over all heads."""
    t = t.to(F64)
    return t / t.pow(2).mean((1, 2), keepdim=True).sqrt()


def o_attention(w, q, k, v, start=0, window=None):
    """q [T, H, D], k [N, G, D], v [N, G, V] -> [T, H*V]"""
    f = lambda t: t.to("cpu", F64)
    R = w.heads // w.kv_heads
    return torch.cat([oracle.sigmoid_attention(
        f(q)[:, h], f(k)[:, h // R], f(v)[:, h // R], w.scale, w.softcap,
        f(w.decay)[h], f(w.reach)[h], f(w.bias)[h],
        window or w.window or 1 << 30, start)
        for h in range(w.heads)], -1)


@where
@pytest.mark.parametrize("size", [(6, 2, 24, 40), (3, 1, 9, 7),
                                  (4, 4, 64, 136), (40, 8, 128, 128)],
                         ids=str)
@pytest.mark.parametrize("n", [1, 70])
def test_norm_over_the_whole_projection(where, size, n):
    """Heads of very different magnitude keep their proportions; weights,
    eps; pages in mixed order; strided rows and rows still in parts."""
    dev, dt = where
    H, G, D, V = size
    g, w = attn_params(dev, H, G, D, V, 50)
    loud = lambda h: torch.logspace(-2, 1, h)[:, None]
    q = torch.randn(n, H, D, generator=g) * loud(H)
    k = torch.randn(n, G, D, generator=g) * loud(G).flip(0)
    v = torch.randn(n, G, V, generator=g)
    qn, kn = (1 + 0.3 * torch.randn(m, generator=g) for m in (H * D, G * D))
    eps = 0.5
    rows = torch.cat([t.reshape(n, -1) for t in (q, k, v)], 1)
    forms = {}
    buf = torch.zeros(n, rows.shape[1] + 8, dtype=dt)
    buf[:, :rows.shape[1]] = rows
    forms["rows"] = (buf.to(dev), buf[:, :rows.shape[1]].to(F64))
    if dt == BF16 and dev != "cpu":
        parts = torch.randn(3, *buf.shape, generator=g)
        parts[:, :, :rows.shape[1]] += rows
        forms["parts"] = (ops.Partials(parts.to(dev)),
                          parts[:, :, :rows.shape[1]].to(F64).sum(0))
    for p, exact_rows in forms.values():
        cache = new_cache(dev, dt, w, n + 20)
        other, slot = cache.alloc_slot(), cache.alloc_slot()
        cache.ensure(slot, n // 2)
        cache.ensure(other, 20)
        cache.ensure(slot, n)
        for pool in (cache.key_pool[0], cache.value_pool[0]):
            pool.fill_(3.0)
        sl, pos = rows_of(dev, [slot], [n], [n])
        got = ops.qk_norm_append(p, cache, 0, w, qn.to(dev), kn.to(dev), eps,
                                 sl, pos)
        wq, wk, wv = exact_rows.split([H * D, G * D, G * V], 1)
        wq = oracle.rms_norm(wq, qn.to(F64), eps).view(n, H, D)
        wk = oracle.rms_norm(wk, kn.to(F64), eps).view(n, G, D)
        lim = tol(dt, 1e-6, 4e-3)
        assert rel(got[..., :D], wq) < lim
        assert bool((got[..., D:] == 0).all())
        pages = cache.page_table[slot, :-(-n // 16)].long()
        kp, vp = (t[0][pages].transpose(1, 2).flatten(0, 1)[:n]
                  for t in (cache.key_pool, cache.value_pool))
        assert rel(kp[..., :D], wk) < lim
        assert rel(vp[..., :V], wv.reshape(n, G, V)) < lim
        rest = torch.ones(cache.n_pages + 1, dtype=torch.bool, device=dev)
        rest[pages] = False
        assert bool((cache.key_pool[0][rest] == 3.0).all())
        assert bool((cache.value_pool[0][rest] == 3.0).all())


ATTN_SIZES = [(6, 2, 24, 40), (3, 1, 9, 7), (20, 1, 64, 136),
              (4, 4, 80, 64), (8, 2, 128, 128), (2, 1, 256, 250)]


@where
@pytest.mark.parametrize("size", ATTN_SIZES, ids=str)
@pytest.mark.parametrize("window", [0, 1, 48, 100])
@pytest.mark.parametrize("form", ["whole", "large tiles", "portions",
                                  "single"])
def test_sigmoid_attention(where, size, window, form, monkeypatch):
    """Whole prompts, portions down to two tokens and single tokens over a
    context whose length is no multiple of anything, with pages handed out
    in a mixed order."""
    dev, dt = where
    if form == "large tiles":
        from ollamamq_amd.ops import hip
        monkeypatch.setattr(hip, "ATTN_LARGE", 0)
    H, G, D, V = size
    kv = 130 if form == "single" else 260
    g, w = attn_params(dev, H, G, D, V, window, seed=window)
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
        got.append(ops.sigmoid_attention(qq, cache, 0, w, sl, pos,
                                         meta).cpu())
        at += n
    want = o_attention(w, unit(q), unit(k), v)
    assert rel(torch.cat(got), want) < tol(dt, 3e-6, 1.2e-2)


def fill_pools(cache, slot, k, v):
    """Keys and values straight into the pages, past the norm."""
    n = k.shape[0]
    cache.ensure(slot, n)
    pages = cache.page_table[slot, :-(-n // 16)].long()
    for pool, t in ((cache.key_pool[0], k), (cache.value_pool[0], v)):
        full = torch.zeros(len(pages) * 16, *t.shape[1:], dtype=t.dtype)
        full[:n] = t
        pool[pages, :, :, :t.shape[2]] = full.view(
            -1, 16, *t.shape[1:]).transpose(1, 2).to(pool.device)


def aimed(w, g, kv, marks, dt):
    """Keys at `marks` stand out for every query, each with its own value;
    all other weights are close to zero."""
    k = 0.1 * torch.randn(kv, w.kv_heads, w.dim, generator=g)
    d = torch.randn(w.kv_heads, w.dim, generator=g)
    d /= d.norm(dim=-1, keepdim=True)
    for j in marks:
        k[j] = 4.0 * d
    q = 4.0 * d.repeat_interleave(w.heads // w.kv_heads, 0)
    return q.to(dt), k.to(dt)


@where
@pytest.mark.parametrize("window", [1, 2, 15, 16, 17, 33, 64, 65, 200])
@pytest.mark.parametrize("n", [1, 2, 40])
def test_window_edges(where, window, n):
    """The last key inside and the first key outside each window: one token
    more or less shows, in decoding and in portions."""
    dev, dt = where
    H, G, D, V, kv = 4, 2, 32, 24, 290
    g, w = attn_params(dev, H, G, D, V, window, seed=3, scale=1.0, bias=-8.0)
    for first in (window - 1, 63, 64, 79, 200, kv - n):
        if not 0 <= first <= kv - n:
            continue
        for edge in sorted({first, first + n - 1}):
            inside, outside = edge - window + 1, edge - window
            marks = [j for j in (inside, outside) if j >= 0]
            q1, k = aimed(w, g, kv, marks, dt)
            v = torch.randn(kv, G, V, generator=g).to(dt)
            cache = new_cache(dev, dt, w, kv)
            slot = cache.alloc_slot()
            fill_pools(cache, slot, k, v)
            sl, pos = rows_of(dev, [slot], [n], [first + n])
            meta = meta_for(dev, [slot], [n], [first + n])
            got = ops.sigmoid_attention(
                q1.expand(n, H, D).contiguous().to(dev), cache, 0, w, sl,
                pos, meta).cpu()
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
    g, w = attn_params(dev, H, G, D, V, 0, seed=5, scale=1.0, bias=-6.0)
    for j in (0, 1, 15, 16, 31, 32, 63, 64, 65, 127, 128, 255, 256, 399,
              kv - n):
        q1, k = aimed(w, g, kv, [j], dt)
        v = torch.randn(kv, G, V, generator=g).to(dt)
        cache = new_cache(dev, dt, w, kv)
        slot = cache.alloc_slot()
        fill_pools(cache, slot, k, v)
        sl, pos = rows_of(dev, [slot], [n], [kv])
        got = ops.sigmoid_attention(
            q1.expand(n, H, D).contiguous().to(dev), cache, 0, w, sl, pos,
            meta_for(dev, [slot], [n], [kv])).cpu()
        want = o_attention(w, q1.expand(n, H, D), k, v, kv - n)
        cos = torch.cosine_similarity(want[-1, :V], v[j, 0].to(F64), 0)
        assert cos > 0.9, "the aimed key must stand out"
        assert rel(got, want) < tol(dt, 1e-5, 2e-2), j


@where
@pytest.mark.parametrize("softcap", [0.0, 0.5, 4.0, 1000.0])
def test_score_cap(where, softcap):
    """Scores from far below to far above the cap; 0 is no cap."""
    dev, dt = where
    H, G, D, V, kv = 4, 2, 32, 32, 90
    g, w = attn_params(dev, H, G, D, V, 50, seed=9, scale=1.0,
                       softcap=softcap)
    q, k = (torch.randn(kv, h, D, generator=g).to(dt) for h in (H, G))
    v = torch.randn(kv, G, V, generator=g).to(dt)
    cache = new_cache(dev, dt, w, kv)
    qq, sl, pos, meta = put_kv(cache, w, cache.alloc_slot(), 0, q, k, v)
    got = ops.sigmoid_attention(qq, cache, 0, w, sl, pos, meta)
    ref = w if softcap else w._replace(softcap=1e9)
    want = o_attention(ref, unit(q), unit(k), v)
    if 0 < softcap < 5:
        assert rel(o_attention(w._replace(softcap=1e9), unit(q), unit(k), v),
                   want) > 0.05
    assert rel(got, want) < tol(dt, 3e-6, 1.5e-2)


@where
def test_long_distances(where):
    """The penalty over thousands of tokens, decoded with the context split
    over blocks."""
    dev, dt = where
    H, G, D, V, kv = 2, 1, 16, 16, 5000
    g, w = attn_params(dev, H, G, D, V, 4500, seed=2, bias=2.0)
    q, k = (torch.randn(kv, h, D, generator=g).to(dt) for h in (H, G))
    v = (1 + torch.randn(kv, G, V, generator=g)).to(dt)
    cache = new_cache(dev, dt, w, kv)
    slot = cache.alloc_slot()
    put_kv(cache, w, slot, 0, q[:-1], k[:-1], v[:-1])
    qq, sl, pos, meta = put_kv(cache, w, slot, kv - 1, q[-1:], k[-1:],
                               v[-1:])
    got = ops.sigmoid_attention(qq, cache, 0, w, sl, pos, meta)
    want = o_attention(w, unit(q[-1:]), unit(k), v, kv - 1)
    assert rel(got, want) < tol(dt, 3e-6, 5e-3)


def moe_case(dev, dt, E, top, K, F, N, T, seed=0, hot=None):
    """hot: the expert that nearly every token chooses first."""
    g = torch.Generator().manual_seed(seed)
    m = lambda n, k: (torch.randn(n, k, generator=g) / k ** 0.5).to(BF16)
    router = m(E, K) * 2
    h = torch.randn(T, K, generator=g)
    if hot is not None:
        h[: T - T // 8] += 2 * router[hot].float() * K ** 0.5
    experts = [(m(F, K), m(F, K), m(N, F)) for _ in range(E)]
    put = lambda t: t.to(dev, dt)
    return h.to(dt), router, experts, ops.moe_weights(put(router), experts,
                                                      top, put)


def o_experts(h, experts, chosen):
    out = torch.zeros(*chosen.shape, experts[0][2].shape[0], dtype=F64)
    for t in range(h.shape[0]):
        for s, e in enumerate(chosen[t].tolist()):
            out[t, s] = oracle.expert(h[t].to(F64),
                                      *(m.to(F64) for m in experts[e]))
    return out


@where
@pytest.mark.parametrize("E,top,K", [(1, 1, 64), (5, 2, 90), (16, 16, 128),
                                     (70, 6, 2048), (8, 1, 96)])
def test_router(where, E, top, K):
    """Choice, order and shares, which sum to less than one unless every
    expert is chosen."""
    dev, dt = where
    h, router, _, w = moe_case(dev, dt, E, top, K, 8, 8, 37)
    chosen, share = ops.moe_route(h.to(dev), w)
    z = h.to(F64) @ router.to(F64).T
    want_e, want_s = oracle.route(h.to(F64), router.to(F64), top)
    assert rel(share, want_s) < 1e-5
    gap = (z.sort(-1, descending=True).values.diff(dim=-1).abs()
           .min(-1).values if E > 1 else torch.ones(37))
    clear = gap > 1e-4
    assert clear.sum() > 20
    assert bool((chosen.cpu().long() == want_e)[clear].all())
    if top < E:
        assert bool((share.sum(-1) < 1).all())


@where
@pytest.mark.parametrize("size", [(5, 2, 64, 48, 64), (3, 3, 90, 34, 90),
                                  (9, 4, 128, 200, 130), (2, 1, 192, 64, 64)],
                         ids=str)
@pytest.mark.parametrize("T", [1, 2, 31, 300])
def test_experts(where, size, T):
    """One token to more than a tile for every expert; a hot expert and idle
    ones."""
    dev, dt = where
    E, top, K, F, N = size
    for hot in (None, E - 1):
        h, router, experts, w = moe_case(dev, dt, E, top, K, F, N, T, T, hot)
        chosen, share = ops.moe_route(h.to(dev), w)
        want = o_experts(h, experts, chosen)
        packs = {"gate_up": ops.pack_weight(w.gate_up.flatten(0, 1)),
                 "down": ops.pack_weight(w.down.flatten(0, 1))}
        for pk in ({}, {k: p for k, p in packs.items() if p is not None}):
            got = ops.moe_experts(h.to(dev), w, chosen, share, pk)
            assert rel(got.parts, want) < tol(dt, 2e-6, 8e-3)
            assert torch.equal(got.share, share)


@GPU
@pytest.mark.parametrize("T", [1, 5, 32, 33, 64])
@pytest.mark.parametrize("size", [(5, 2, 64, 64, 64), (3, 3, 192, 100, 96),
                                  (40, 7, 128, 64, 128), (2, 1, 2112, 64, 32)],
                         ids=str)
def test_streamed_experts(T, size):
    """The decode form: packed weights, activations in fragment layout."""
    E, top, K, F, N = size
    for hot in (None, 0):
        h, router, experts, w = moe_case("cuda:0", BF16, E, top, K, F, N, T,
                                         T, hot)
        # the row kernel makes the layout
        _, hf = ops.rms_residual(h.float().cuda(), None, None, None, 1.0,
                                 0.0, embed=h.cuda(), frag=True)
        chosen, share = ops.moe_route(hf, w)
        plain, share2 = ops.moe_route(h.cuda(), w)
        assert torch.equal(chosen, plain) and torch.equal(share, share2)
        # and chooses on the way, if there are few experts
        y, post = torch.zeros_like(h).cuda(), torch.ones(K, device="cuda")
        for z in (y, ops.Partials(y.float()[None])):
            x2, h2, (chosen3, share3) = ops.rms_residual_route(
                h.float().cuda(), z, post, 1.0, 1.0, w, embed=h.cuda(),
                frag=True)
            assert torch.equal(x2.cpu(), h.float())
            assert torch.equal(chosen3, chosen)
            assert rel(share3, share.cpu()) < 1e-5
        packs = {"gate_up": ops.pack_weight(w.gate_up.flatten(0, 1)),
                 "down": ops.pack_weight(w.down.flatten(0, 1))}
        got = ops.moe_experts(hf, w, chosen, share, packs)
        assert rel(got.parts, o_experts(h, experts, chosen)) < 8e-3


# --------------------------------------------------------------- whole models

def test_config_reaches_every_constant(models):
    _, cfg, _ = models["mixed"]
    rc = RevitarConfig.from_json(cfg)
    assert (rc.eps, rc.embed_scale, rc.residual_mult) == (1e-5, 0.6, 0.4)
    a, b, c = rc.layers
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.window) == (6, 2, 24, 40,
                                                              37)
    assert (a.experts, a.top, a.ff, b.ff, c.top) == (5, 2, 80, 0, 1)
    assert (a.softcap, c.softcap) == (15.0, 2.0)
    assert [s.kv for s in rc.run_stores()] == [(2, 24, 40), (4, 48, 16),
                                               (1, 16, 72)]


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
@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_greedy_generation(models, where, name):
    """Through submit/step: admission, chunked prompts, mixed steps, the
    pipelined decode, slots that are freed and taken again.  Every token is
    the oracle's argmax (or a tie within rounding)."""
    dev, dt = where
    path, cfg, w = models[name]
    rc = config_from_folder(path)
    kv = cache_for_model(rc, n_pages=40, max_slots=3, max_ctx=160,
                         device=dev, dtype=dt)
    eng = LlamaEngine(build_model(rc, device=dev, dtype=dt), kv, max_batch=3,
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
    rc = config_from_folder(path)

    def run(graphs):
        kv = cache_for_model(rc, n_pages=64, max_slots=6, max_ctx=160,
                             device="cuda:0", dtype=dt)
        eng = LlamaEngine(build_model(rc, device="cuda:0", dtype=dt), kv,
                          max_batch=6)
        assert eng.model.frag_decode == (dt == BF16)
        eng.use_graphs = eng.use_pipeline = graphs
        if graphs:
            eng.warm_graphs()
        return generate(eng, [tokens_for(name, n, n) for n in
                              (3, 20, 9, 14, 30)], 25)

    assert run(True) == run(False)


@where
def test_preset_runs(where):
    dev, dt = where
    from ollamamq_amd.models import PRESETS
    cfg = PRESETS["revitar-tiny"]
    kv = cache_for_model(cfg, n_pages=32, max_slots=2, max_ctx=128,
                         device=dev, dtype=dt)
    model = build_model(cfg, device=dev, dtype=dt, seed=3)
    eng = LlamaEngine(model, kv, max_batch=2)
    out = generate(eng, [[1, 2, 3], [4] * 20], 5)
    assert all(len(o) == 5 for o in out)
    assert len(eng.embed([1, 2, 3])) == cfg.width
    assert cfg.model_info()["expert_used_count"] == 2


# ------------------------------------------------------------ loading, runner

def test_bad_checkpoints_are_refused(models, tmp_path):
    path, cfg, w = models["odd"]
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    bad = dict(w)
    bad["l1.mlp.e2.up"] = torch.zeros(3, 90, dtype=BF16)
    save_file(bad, str(tmp_path / "model.safetensors"))
    with pytest.raises(ValueError, match="l1.mlp.e2.up"):
        build_model(config_from_folder(str(tmp_path)))
    del bad["l1.mlp.e2.up"]
    save_file(bad, str(tmp_path / "model.safetensors"))
    with pytest.raises(KeyError, match="l1.mlp.e2.up"):
        build_model(config_from_folder(str(tmp_path)))

    def changed(**kw):
        other = json.loads(json.dumps(cfg))
        other["layers"][0].update(kw)
        return RevitarConfig.from_json(other)

    with pytest.raises(ValueError, match="something"):
        changed(type="something")
    with pytest.raises(ValueError, match="dense"):
        changed(mlp={"kind": "dense", "ff": 3})
    with pytest.raises(ValueError, match="evenly"):
        changed(mixer={**cfg["layers"][0]["mixer"], "kv_heads": 2})
    with pytest.raises(ValueError, match="top 3"):
        changed(mlp={"kind": "moe", "expert": {"ff": 8},
                     "router": {"experts": 2, "top": 3}})
    with pytest.raises(ValueError, match="parallel"):
        build_model(RevitarConfig.from_json(cfg), tp_size=2)


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
    register_checkpoint(f"experts-folder={models['mixed'][0]}")
    try:
        w = Worker(0, max_batch=2, default_ctx=128)
        assert "experts-folder" in w.available_models()
        q = queue.Queue()
        w.generate("experts-folder", [1, 2, 3], GenParams(max_tokens=6),
                   lambda t, done: q.put((t, done)))
        out = []
        while True:
            t, done = q.get(timeout=60)
            if done:
                break
            out.append(t)
        assert len(out) == 6
        assert w.unload("experts-folder") is None
    finally:
        PRESETS.pop("experts-folder")
