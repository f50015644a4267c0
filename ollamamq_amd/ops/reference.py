"""Plain-PyTorch fp32 reference implementations of every hot op.

These are the numerics oracle for the gfx950 HIP kernels (tests compare the
HIP path against these at fp32) and the CPU execution path for the
dispatcher/scheduler test suite, which runs with no GPU (the
reference's whole test strategy runs on loopback without real backends).
"""
from __future__ import annotations

import math

import torch


def rmsnorm_residual(x, residual, weight, eps):
    """y = rmsnorm(x + residual) * weight; returns (y, x + residual).

    residual may be None (plain rmsnorm). Always accumulates in fp32.
    """
    if residual is not None:
        residual = (x.float() + residual.float())
    else:
        residual = x.float()
    var = residual.pow(2).mean(dim=-1, keepdim=True)
    y = residual * torch.rsqrt(var + eps) * weight.float()
    return y.to(x.dtype), residual.to(x.dtype)


def rope(q, k, positions, cos, sin):
    """In-place NeoX-style half-rotation RoPE on q [T,Hq,D] and k [T,Hk,D].

    cos/sin: [max_ctx, D/2] host-precomputed tables (guide Appendix B:
    on-device trig turns a memory-bound op VALU-bound).
    """
    c = cos[positions.long()].unsqueeze(1)  # [T,1,D/2]
    s = sin[positions.long()].unsqueeze(1)
    for t in (q, k):
        d2 = t.shape[-1] // 2
        # NB: .float() on an fp32 tensor is a VIEW — compute both halves
        # before mutating t, or the lower-half store corrupts x1.
        x1 = t[..., :d2].float()
        x2 = t[..., d2:].float()
        lo = x1 * c - x2 * s
        hi = x2 * c + x1 * s
        t[..., :d2] = lo.to(t.dtype)
        t[..., d2:] = hi.to(t.dtype)


def kv_append(cache, layer, k, v, slot_ids, positions):
    """Scatter k/v [T, KVH, D] into the paged pool at (slot, position)."""
    ps = cache.page_size
    pages = cache.page_table[slot_ids.long(), (positions // ps).long()]
    offs = (positions % ps).long()
    cache.k_pool[layer, pages.long(), :, offs] = k.to(cache.k_pool.dtype)
    cache.v_pool[layer, pages.long(), :, offs] = v.to(cache.v_pool.dtype)


def _gather_kv(cache, layer, slot, kv_len):
    """Return K,V [kv_len, KVH, D] for one slot from the paged pool."""
    ps = cache.page_size
    n_pages = (kv_len + ps - 1) // ps
    pages = cache.page_table[slot, :n_pages].long()
    k = cache.k_pool[layer, pages]  # [n_pages, KVH, ps, D]
    v = cache.v_pool[layer, pages]
    k = k.permute(0, 2, 1, 3).reshape(n_pages * ps, -1, cache.head_dim)
    v = v.permute(0, 2, 1, 3).reshape(n_pages * ps, -1, cache.head_dim)
    return k[:kv_len], v[:kv_len]


def attention(q, cache, layer, meta):
    """Causal paged attention, prefill (varlen) and decode alike.

    q: [T, Hq, D] flat over sequences; meta gives per-sequence q extents.
    Query token at absolute position p attends KV positions [0, p].
    GQA: Hq queries share Hq/Hkv groups. fp32 math throughout.
    """
    T, Hq, D = q.shape
    out = torch.empty_like(q)
    scale = 1.0 / (D ** 0.5)
    cu = meta.cu_q.tolist()
    slots = meta.slot_ids.tolist()
    lens = meta.seq_lens.tolist()
    for i, slot in enumerate(slots):
        q_i = q[cu[i]:cu[i + 1]].float()          # [qlen, Hq, D]
        qlen = q_i.shape[0]
        kv_len = lens[i]
        k, v = _gather_kv(cache, layer, slot, kv_len)
        k = k.float()
        v = v.float()
        rep = Hq // k.shape[1]
        k = k.repeat_interleave(rep, dim=1)       # [kv, Hq, D]
        v = v.repeat_interleave(rep, dim=1)
        scores = torch.einsum("qhd,khd->hqk", q_i, k) * scale
        # causal: query j sits at absolute position kv_len - qlen + j
        qpos = torch.arange(kv_len - qlen, kv_len, device=q.device)
        kpos = torch.arange(kv_len, device=q.device)
        mask = kpos[None, :] > qpos[:, None]
        if meta.window and meta.window > 0:
            # sliding window: query p attends [max(0, p-window+1), p]
            mask |= kpos[None, :] < qpos[:, None] - meta.window + 1
        scores.masked_fill_(mask.unsqueeze(0), float("-inf"))
        p = torch.softmax(scores, dim=-1)
        o = torch.einsum("hqk,khd->qhd", p, v)
        out[cu[i]:cu[i + 1]] = o.to(q.dtype)
    return out


def swiglu(gate_up, act="silu"):
    """[T, 2F] fused gate/up -> act(gate) * up, fp32 math."""
    f = gate_up.shape[-1] // 2
    g = gate_up[..., :f].float()
    u = gate_up[..., f:].float()
    g = {"silu": torch.nn.functional.silu,
         "gelu_tanh": lambda t: torch.nn.functional.gelu(
             t, approximate="tanh")}[act](g)
    return (g * u).to(gate_up.dtype)


def dyt_residual(x, y, post, pre, shift, embed, tokens, rows):
    if x is None:
        x = embed.index_select(0, tokens.long()).float()
    if y is not None:
        x = x + torch.tanh(post.alpha * y.float()) * post.w + post.b
    if rows is not None:
        x = x[rows]
    h = torch.tanh(pre.alpha * x) * pre.w + pre.b
    if shift is not None:
        before = torch.roll(h, 1, 0)
        slots, q_lens, _ = shift.meta.layout()
        r = 0
        for slot, n in zip(slots, q_lens):
            before[r] = 0 if shift.positions[r] == 0 else shift.prev[slot]
            shift.prev[slot] = h[r + n - 1]
            r += n
        h = h + (before - h) * shift.mix
    return x, h.to(embed.dtype if embed is not None else pre.w.dtype)


def polynorm(z, coef, eps):
    f = z.float()
    out = torch.full_like(f, coef[3])
    for k in range(3):
        p = f ** (k + 1)
        out += coef[k] * p * torch.rsqrt(p.pow(2).mean(-1, True) + eps)
    return out.to(z.dtype)


def latent_append(cache, run, d, weight, slot_ids, positions, eps):
    f = d.float()
    c = f * torch.rsqrt(f.pow(2).mean(-1, True) + eps) * weight
    ps = cache.page_size
    pages = cache.page_table[slot_ids.long(), (positions // ps).long()]
    pool = cache.latent_pool[run]
    pool[pages.long(), (positions % ps).long()] = c.to(pool.dtype)


def whole(p):
    """A projection in fp32, its partial sums added up."""
    return p.parts.sum(0) if hasattr(p, "parts") else p.float()


def _rotate(x, positions, rope):
    """The pairs of x [T, H, dim], fp32."""
    if not rope.dims:
        return x
    cs = rope.table[positions.long()].unsqueeze(1)       # [T, 1, dims]
    c, s = cs[..., 0::2], cs[..., 1::2]
    if rope.halves:
        u, v = x[..., :rope.dims].chunk(2, -1)
    else:
        u, v = x[..., 0:rope.dims:2], x[..., 1:rope.dims:2]
    turned = [u * c - v * s, v * c + u * s]
    turned = torch.cat(turned, -1) if rope.halves \
        else torch.stack(turned, -1).flatten(-2)
    return torch.cat([turned, x[..., rope.dims:]], -1)


def latent_rope_append(p, cache, run, w, norm, eps, rope, slot_ids,
                       positions):
    H, D, R = w.uk.shape
    E, f, T = w.rot_dim, whole(p), slot_ids.shape[0]
    q, c, k = f[:, :H * (D + E) + R + E].split([H * (D + E), R, E], 1)
    q = q.reshape(T, H, D + E)
    q = torch.cat([q[..., :D], _rotate(q[..., D:], positions, rope)], -1)
    pool, ps = cache.latent_pool[run], cache.page_size
    pages = cache.page_table[slot_ids.long(), (positions // ps).long()]
    row = torch.cat([_unit_rms(c, eps) * norm,
                     _rotate(k.unsqueeze(1), positions, rope).squeeze(1)], -1)
    pool[pages.long(), (positions % ps).long(), :R + E] = row.to(pool.dtype)
    return q.reshape(T, -1).to(pool.dtype)


def latent_attention(q, cache, run, w, meta, gate=None):
    H, D, R = w.uk.shape
    T, E = q.shape[0], w.rot_dim
    pool = cache.latent_pool[run]
    out = torch.empty(T, H, w.uv.shape[1], dtype=q.dtype, device=q.device)
    r = 0
    for slot, n, kv in zip(*meta.layout()):
        pages = cache.page_table[slot, :-(-kv // cache.page_size)].long()
        row = pool[pages].flatten(0, 1)[:kv].float()
        c = row[:, :R]
        k = torch.einsum("tr,hdr->htd", c, w.uk.float())
        k = torch.cat([k, row[:, R:R + E].expand(H, kv, E)], -1)
        v = torch.einsum("tr,hvr->htv", c, w.uv.float())
        qi = q[r:r + n].float().view(n, H, D + E).transpose(0, 1)
        s = qi @ k.transpose(1, 2) * w.scale
        s.masked_fill_(~_seen(n, kv, w.window), float("-inf"))
        out[r:r + n] = (torch.softmax(s, -1) @ v).transpose(0, 1)
        r += n
    out = out.view(T, -1)
    if gate is not None:
        g = whole(gate.p)[:, gate.first:gate.first + out.shape[1]]
        out = (out.float() * torch.sigmoid(g)).to(out.dtype)
    return out


def _seen(n, kv, window, chunk=0):
    """Keys that the last n of kv tokens see."""
    i, j = torch.arange(kv - n, kv)[:, None], torch.arange(kv)[None]
    seen = (j <= i) & (i - j < (window or kv))
    return seen & (i // chunk == j // chunk) if chunk else seen


def rope_qkv_append(p, bias, cache, run, w, rope, slot_ids, positions):
    f = whole(p)[:, :w.heads * w.dim + w.kv_heads * (w.dim + w.vdim)]
    if bias is not None:
        f = f + bias
    return _append(*_split_heads(f, w), cache, run, rope, slot_ids,
                   positions)


def _split_heads(f, w):
    """Columns q | k | v as [T, heads, width] each."""
    H, G, D, V = w.heads, w.kv_heads, w.dim, w.vdim
    T = f.shape[0]
    q, k, v = f[:, :H * D + G * (D + V)].split([H * D, G * D, G * V], -1)
    return q.reshape(T, H, D), k.reshape(T, G, D), v.reshape(T, G, V)


def _append(q, k, v, cache, run, rope, slot_ids, positions):
    """Rotate queries and keys, append keys and values."""
    D, V = k.shape[2], v.shape[2]
    kp, vp = cache.key_pool[run], cache.value_pool[run]
    ps = cache.page_size
    pages = cache.page_table[slot_ids.long(), (positions // ps).long()].long()
    offs = (positions % ps).long()
    kp[pages, :, offs, :D] = _rotate(k, positions, rope).to(kp.dtype)
    vp[pages, :, offs, :V] = v.to(vp.dtype)
    out = torch.zeros(*q.shape[:2], kp.shape[3], dtype=kp.dtype,
                      device=kp.device)
    out[:, :, :D] = _rotate(q, positions, rope)
    return out


def qkv_norm_rope_append(p, norms, cache, run, w, rope, slot_ids, positions):
    q, k, v = _split_heads(whole(p), w)
    q, k = _unit_rms(q, norms.eps) * norms.q, _unit_rms(k, norms.eps) * norms.k
    if norms.gain is not None:
        q = q * norms.gain[:, None]
    if norms.values:
        v = _unit_rms(v, norms.eps)
    return _append(q, k, v, cache, run, rope, slot_ids, positions)


def softmax_attention(q, cache, run, w, meta, gate=None):
    T, H, G, V = q.shape[0], w.heads, w.kv_heads, w.vdim
    kp, vp = cache.key_pool[run], cache.value_pool[run]
    out = torch.empty(T, H, V, dtype=q.dtype, device=q.device)
    r = 0
    for slot, n, kv in zip(*meta.layout()):
        pages = cache.page_table[slot, :-(-kv // cache.page_size)].long()
        k, v = (pool[pages].transpose(1, 2).flatten(0, 1)[:kv].float()
                .repeat_interleave(H // G, 1).transpose(0, 1)
                for pool in (kp, vp))
        s = q[r:r + n].float().transpose(0, 1) @ k.transpose(1, 2) * w.scale
        s.masked_fill_(~_seen(n, kv, w.window, w.chunk), float("-inf"))
        if w.sink is not None:
            s = torch.cat([s, w.sink.view(H, 1, 1).expand(H, n, 1)], -1)
        a = torch.softmax(s, -1)[..., :kv]
        out[r:r + n] = (a @ v)[..., :V].transpose(0, 1)
        r += n
    if gate is not None:
        g = whole(gate.p)[:, gate.first:gate.first + H]
        out = (out.float() * torch.sigmoid(g)[..., None]).to(out.dtype)
    return out.view(T, H * V)


def _gated_heads(o, norm, gate, eps, dtype, per_head=True, act="sigmoid"):
    """Norm of o [T, H, V], of every head or of all together, and the output
    gate [T, H*V]."""
    T, H, V = o.shape
    o = _unit_rms(o if per_head else o.reshape(T, 1, H * V), eps) \
        .reshape(T, H * V)
    if norm is not None:
        o = o * norm.repeat(H * V // norm.numel())
    g = torch.sigmoid(gate) if act == "sigmoid" \
        else torch.nn.functional.silu(gate)
    return (o * g).to(dtype)


def _type_of(p):
    return p.dtype if torch.is_tensor(p) else torch.bfloat16


def lightning(p, w, state, meta):
    H, D, V = w.heads, w.dim, w.vdim
    oq, ok, ov, og = w.offsets
    f = whole(p)
    T = f.shape[0]
    act = torch.nn.functional.silu if w.act else lambda t: t
    part = lambda at, n: act(f[:, at:at + H * n]).view(T, H, n)
    q, k, v = part(oq, D), part(ok, D), part(ov, V)
    decay = w.powers[:, 1].view(H, 1, 1)
    out = torch.empty(T, H, V)
    r = 0
    for slot, n, kv in zip(*meta.layout()):
        S = state[slot] if kv > n else torch.zeros_like(state[slot])
        for t in range(r, r + n):
            S = decay * S + k[t].unsqueeze(-1) * v[t].unsqueeze(1)
            out[t] = torch.einsum("hdv,hd->hv", S, q[t])
        state[slot] = S
        r += n
    return _gated_heads(out * w.scale, w.norm, f[:, og:og + H * V], w.eps,
                        _type_of(p), w.per_head, w.gate)


def _delta(q, k, v, z, e, g, state, meta):
    """S <- diag(g) S - e (z^T S) + k v^T with the old state on the right,
    o = S^T q; everything [T, H, D] but v."""
    out = torch.empty(v.shape)
    r = 0
    for slot, n, kv in zip(*meta.layout()):
        S = state[slot] if kv > n else torch.zeros_like(state[slot])
        for t in range(r, r + n):
            read = torch.einsum("hdv,hd->hv", S, z[t])
            S = g[t].unsqueeze(-1) * S - e[t].unsqueeze(-1) \
                * read.unsqueeze(1) + k[t].unsqueeze(-1) * v[t].unsqueeze(1)
            out[t] = torch.einsum("hdv,hd->hv", S, q[t])
        state[slot] = S
        r += n
    return out


def _unit(x):
    from .interface import UNIT_EPS
    return x * torch.rsqrt(x.pow(2).sum(-1, True) + UNIT_EPS)


def _short_conv(x, w, state, meta):
    """x [T, C], w [taps, C]; state [slots, taps - 1, C] holds a sequence's
    last inputs."""
    taps = w.shape[0]
    out = torch.empty_like(x)
    r = 0
    for slot, n, kv in zip(*meta.layout()):
        before = state[slot] if kv > n else torch.zeros_like(state[slot])
        row = torch.cat([before, x[r:r + n]])
        out[r:r + n] = sum(row[j:j + n] * w[j] for j in range(taps))
        state[slot] = row[n:]
        r += n
    return out


def gated_delta(p, w, state, conv_state, meta):
    H, G, D, V = w.heads, w.kv_heads, w.dim, w.vdim
    o_in, ob, oa, og = w.offsets
    f = whole(p)
    T, C = f.shape[0], w.conv.shape[1]
    y = torch.nn.functional.silu(_short_conv(f[:, o_in:o_in + C], w.conv,
                                             conv_state, meta))
    q, k, v = y.split([G * D, G * D, H * V], -1)
    heads = lambda t: _unit(t.reshape(T, G, D)).repeat_interleave(H // G, 1)
    q, k, v = heads(q) * D ** -0.5, heads(k), v.reshape(T, H, V)
    low = lambda at, m: f[:, at:at + m.rank] @ m.w.float().T
    z = torch.nn.functional.softplus(low(oa, w.a2) + w.dt_bias)
    g = torch.exp(-w.rate[:, None] * z.view(T, H, D))
    bk = torch.sigmoid(f[:, ob:ob + H]).unsqueeze(-1) * k
    o = _delta(q, bk, v, g * k, bk, g, state, meta)
    return _gated_heads(o, w.norm, low(og, w.g2), w.eps, _type_of(p))


def general_delta(p, w, state, meta):
    H, D = w.heads, w.dim
    f = whole(p)
    T = f.shape[0]
    r, k, v, a, gate = (f[:, at:at + H * D] for at in w.offsets[:5])
    heads = lambda t: t.reshape(T, H, D)
    u = _unit(heads(k))
    at = w.offsets[5]
    z = torch.tanh(f[:, at:at + w.w2.rank]) @ w.w2.w.float().T + w.w0
    g = torch.exp(-math.exp(-0.5) * torch.sigmoid(z))
    a = torch.sigmoid(a + w.a_bias)
    o = _delta(heads(r), heads(k), heads(v), u, heads(a) * u, heads(g), state,
               meta)
    return _gated_heads(o, w.norm, gate, w.eps, _type_of(p))


def _layer_norm(x, norm, eps):
    return torch.nn.functional.layer_norm(x, x.shape[-1:], norm.w, norm.b,
                                          eps)


def ln_residual(x, y, norm, mult, eps, scale, embed, tokens, rows, then):
    if x is None:
        x = embed.index_select(0, tokens.long()).float()
    if y is not None:
        if hasattr(y, "pairs"):
            y = y.share * sum(_unit_rms(whole(b), eps) * w
                              for b, w in y.pairs)
        y = whole(y)
        x = _layer_norm(mult * x + (y if scale is None else scale * y), norm,
                        eps)
    if rows is not None:
        x = x[rows]
    h = x if then is None else _layer_norm(x, then, eps)
    return x, h.to(embed.dtype)


def gla(p, w, state, meta):
    T, H, D, V = p.shape[0], w.heads, w.dim, w.vdim
    oq, ok, ov, og, ou = w.offsets
    f = p.float()
    q = f[:, oq:oq + H * D].view(T, H, D) * D ** -0.5
    k = f[:, ok:ok + H * D].view(T, H, D)
    v = f[:, ov:ov + H * V].view(T, H, V)
    z = f[:, ou:ou + w.rank] @ w.a2.float().T + w.a2_b
    a = torch.exp(torch.nn.functional.logsigmoid(z) / w.tau).view(T, H, D)
    out = torch.empty(T, H, V)
    r = 0
    for slot, n, kv in zip(*meta.layout()):
        S = state[slot] if kv > n else torch.zeros_like(state[slot])
        for t in range(r, r + n):
            S = a[t].unsqueeze(-1) * S + k[t].unsqueeze(-1) * v[t].unsqueeze(1)
            out[t] = torch.einsum("hdv,hd->hv", S, q[t])
        state[slot] = S
        r += n
    out = out * torch.rsqrt(out.pow(2).mean(-1, True) + w.eps) * w.norm
    g = torch.nn.functional.silu(f[:, og:og + H * V]).view(T, H, V)
    return (out * g).reshape(T, H * V).to(p.dtype)


def _unit_rms(x, eps):
    return x * torch.rsqrt(x.pow(2).mean(-1, True) + eps)


def rms_residual(x, y, post, pre, mult, eps, embed, tokens, embed_scale,
                 rows, shift=None, tail=False, bare=False):
    if x is None:
        x = 0.0 if bare else \
            embed.index_select(0, tokens.long()).float() * embed_scale
    if y is not None:
        if hasattr(y, "share"):
            y = (y.parts.float() * y.share.unsqueeze(-1)).sum(1)
        y = whole(y)
        x = x + mult * (y if post is None else _unit_rms(y, eps) * post)
    if shift is not None:
        x = x + shift
    if rows is not None:
        x = x[rows]
    h = x if pre is None else _unit_rms(x, eps) * pre
    if tail:
        at = tokens if rows is None else tokens[rows]
        h = torch.cat([h, embed.index_select(0, at.long()).float()
                       * embed_scale], -1)
    return x, h.to(embed.dtype)


def qk_norm_append(p, cache, run, w, q_norm, k_norm, eps, slot_ids,
                   positions):
    T, H, G, D, V = p.shape[0], w.heads, w.kv_heads, w.dim, w.vdim
    q, k, v = p[:, :H * D + G * (D + V)].float().split(
        [H * D, G * D, G * V], -1)
    kp, vp = cache.key_pool[run], cache.value_pool[run]
    ps = cache.page_size
    pages = cache.page_table[slot_ids.long(), (positions // ps).long()].long()
    offs = (positions % ps).long()
    k = (_unit_rms(k, eps) * k_norm).view(T, G, D)
    kp[pages, :, offs, :D] = k.to(kp.dtype)
    vp[pages, :, offs, :V] = v.reshape(T, G, V).to(vp.dtype)
    out = torch.zeros(T, H, kp.shape[3], dtype=kp.dtype, device=p.device)
    out[:, :, :D] = (_unit_rms(q, eps) * q_norm).view(T, H, D)
    return out


def sigmoid_attention(q, cache, run, w, meta):
    T, H, G, V = q.shape[0], w.heads, w.kv_heads, w.vdim
    kp, vp = cache.key_pool[run], cache.value_pool[run]
    out = torch.empty(T, H, V, dtype=q.dtype, device=q.device)
    col = lambda t: t.view(H, 1, 1)
    r = 0
    for slot, n, kv in zip(*meta.layout()):
        pages = cache.page_table[slot, :-(-kv // cache.page_size)].long()
        k, v = (pool[pages].transpose(1, 2).flatten(0, 1)[:kv].float()
                .repeat_interleave(H // G, 1).transpose(0, 1)
                for pool in (kp, vp))
        s = q[r:r + n].float().transpose(0, 1) @ k.transpose(1, 2) * w.scale
        if w.softcap > 0:
            s = w.softcap * torch.tanh(s / w.softcap)
        dist = (torch.arange(kv - n, kv)[:, None]
                - torch.arange(kv)[None]).float()
        s = s - col(w.decay) * torch.log1p(col(w.reach) * dist.clamp(min=0))
        a = torch.sigmoid(s + col(w.bias))
        seen = (dist >= 0) & (dist < (w.window or kv))
        out[r:r + n] = ((a * seen) @ v)[..., :V].transpose(0, 1)
        r += n
    return out.view(T, H * V)


def moe_route(h, w):
    share = torch.softmax(h.float() @ w.router.float().T, -1)
    share, chosen = share.topk(w.top, -1)
    return chosen.int(), share


def moe_experts(h, w, chosen, share):
    E, F2, K = w.gate_up.shape
    out = torch.zeros(*chosen.shape, w.down.shape[1])
    for e in range(E):
        t, s = (chosen == e).nonzero(as_tuple=True)
        if len(t):
            gu = (h[t].float() @ w.gate_up[e].float().T).view(
                -1, F2 // 32, 2, 16)
            a = torch.nn.functional.silu(gu[:, :, 0]) * gu[:, :, 1]
            out[t, s] = a.flatten(1) @ w.down[e].float().T
    from .interface import Weighted
    return Weighted(out, share)


def sample(logits, temperature, top_k, top_p, generator=None):
    """Per-row sampling: greedy when temperature<=0, else temp/top-k/top-p.

    logits: [B, V]; temperature/top_k/top_p are python scalars (uniform
    across the batch) OR 1-D [B] tensors — each row is filtered by ITS OWN
    top_k/top_p (per-request semantics: mixed sampling params in one batch
    never bleed into each other).  top_k 0 and top_p >= 1 disable the
    respective filter for that row.  Returns [B] int64 token ids.
    """
    B, V = logits.shape
    dev = logits.device
    logits = logits.float()
    if not torch.is_tensor(temperature):
        temperature = torch.full((B,), float(temperature), device=dev)
    if not torch.is_tensor(top_k):
        top_k = torch.full((B,), int(top_k or 0), dtype=torch.long,
                           device=dev)
    if not torch.is_tensor(top_p):
        top_p = torch.full((B,), float(top_p if top_p else 1.0), device=dev)
    top_k = top_k.long()
    greedy = temperature <= 0
    out = torch.empty(B, dtype=torch.long, device=dev)
    if greedy.any():
        out[greedy] = logits[greedy].argmax(dim=-1)
    rest = ~greedy
    if rest.any():
        l = logits[rest] / temperature[rest].unsqueeze(1)
        tk = top_k[rest]
        tp = top_p[rest]
        if bool(((tk > 0) & (tk < V)).any()) or bool((tp < 1.0).any()):
            # one descending sort serves both filters; applying top-k as a
            # post-softmax mask + renormalize is identical to the -inf
            # pre-softmax mask (softmax restricted to a subset)
            sv, si = l.sort(dim=-1, descending=True)
            sp = torch.softmax(sv, dim=-1)
            ar = torch.arange(V, device=dev)
            kk = torch.where(tk > 0, tk.clamp(max=V), torch.full_like(tk, V))
            keep = ar.unsqueeze(0) < kk.unsqueeze(1)          # per-row top-k
            cum = sp.cumsum(dim=-1)
            keep &= (cum - sp) < tp.unsqueeze(1)   # keep token crossing mass
            keep[:, 0] = True                      # never empty a row
            sp = sp * keep
            sp = sp / sp.sum(dim=-1, keepdim=True)
            pick = torch.multinomial(sp, 1, generator=generator).squeeze(1)
            out[rest] = si.gather(1, pick.unsqueeze(1)).squeeze(1)
        else:
            probs = torch.softmax(l, dim=-1)
            out[rest] = torch.multinomial(
                probs, 1, generator=generator).squeeze(1)
    return out
