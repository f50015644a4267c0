"""Plain, slow statement of the Rinitar equations, in float64 on the CPU.

One function per mechanism, written token by token and head by head, with no
cache, no batching and nothing imported from the framework.  The tests
compare the framework with this.  Weights are a dict name -> tensor with the
checkpoint's names; the configuration is the plain config.json dict.
"""
import math

import torch

F64 = torch.float64


def dyt(x, w, b, alpha):
    """Dynamic tanh, element by element: no statistics of x enter."""
    return torch.tanh(alpha * x) * w + b


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def token_shift(h, mix):
    """h [T, W]: every token is moved towards its predecessor's raw h; the
    first token's predecessor is zero."""
    out = torch.empty_like(h)
    prev = torch.zeros_like(h[0])
    for t in range(h.shape[0]):
        out[t] = h[t] + (prev - h[t]) * mix
        prev = h[t]
    return out


def gla_decay(h, a1, a2, a2_b, tau):
    z = (h @ a1.T) @ a2.T + a2_b
    return torch.sigmoid(z) ** (1.0 / tau)


def gla_scan(q, k, v, alpha, state=None):
    """One head's recurrence: q, k, alpha [T, D], v [T, V] -> o [T, V] and
    the last state [D, V]."""
    T, D = q.shape
    S = torch.zeros(D, v.shape[1], dtype=q.dtype) if state is None \
        else state.clone()
    o = torch.empty(T, v.shape[1], dtype=q.dtype)
    for t in range(T):
        S = alpha[t][:, None] * S + k[t][:, None] * v[t][None, :]
        o[t] = S.T @ q[t]
    return o, S


def gla_mixer(h, p, m, eps):
    """p(name) gives the mixer's tensor, m the mixer's sizes."""
    H, D, V = m["heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q = (h @ p("q").T * D ** -0.5).view(T, H, D)
    k = (h @ p("k").T).view(T, H, D)
    v = (h @ p("v").T).view(T, H, V)
    a = gla_decay(h, p("a1"), p("a2"), p("a2.b"), m["tau"]).view(T, H, D)
    heads = []
    for i in range(H):
        o, _ = gla_scan(q[:, i], k[:, i], v[:, i], a[:, i])
        heads.append(unit_rms(o, eps) * p("norm"))
    o = torch.cat(heads, -1)
    g = h @ p("g").T
    return (o * (g * torch.sigmoid(g))) @ p("o").T


def softmax_attention(q, k, v, scale):
    """One head, causal: q, k [T, D], v [T, V]."""
    out = torch.empty(q.shape[0], v.shape[1], dtype=q.dtype)
    for i in range(q.shape[0]):
        s = (k[:i + 1] @ q[i]) * scale
        e = torch.exp(s - s.max())
        out[i] = (e / e.sum()) @ v[:i + 1]
    return out


def latent_mixer(h, p, m, eps):
    H, D, V = m["heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q = (h @ p("q").T).view(T, H, D)
    c = unit_rms(h @ p("dkv").T, eps) * p("dkv.norm")
    k = (c @ p("uk").T).view(T, H, D)
    v = (c @ p("uv").T).view(T, H, V)
    o = torch.cat([softmax_attention(q[:, i], k[:, i], v[:, i], m["scale"])
                   for i in range(H)], -1)
    return o @ p("o").T


def polynorm(z, coef, eps):
    a, b, c, e = coef
    return (a * unit_rms(z, eps) + b * unit_rms(z ** 2, eps)
            + c * unit_rms(z ** 3, eps) + e)


def layer_order(cfg):
    """Indices of the layers in the order they run, loop unrolled."""
    n = len(cfg["layers"])
    lp = cfg.get("loop")
    if not lp:
        return list(range(n))
    body = list(range(lp["start"], lp["stop"]))
    return (list(range(lp["start"])) + body * lp["times"]
            + list(range(lp["stop"], n)))


def run(cfg, weights, tokens):
    """Logits [T, vocab] and the residual stream after every layer run."""
    W = {k: t.to(F64) for k, t in weights.items()}
    eps = cfg["norm"]["eps"]

    def norm(name, x):
        return dyt(x, W[name], W[name + ".b"], W[name + ".alpha"])

    x = W["embed"][torch.as_tensor(tokens)]
    taps = []
    for i in layer_order(cfg):
        L, pre = cfg["layers"][i], f"l{i}."
        mixer = {"gla": gla_mixer, "latent_attention": latent_mixer}[L["type"]]
        h = token_shift(norm(pre + "norm1", x), W[pre + "shift"])
        y = mixer(h, lambda s: W[pre + "mix." + s], L["mixer"], eps)
        x = x + norm(pre + "norm1b", y)
        if L.get("mlp"):
            h = norm(pre + "norm2", x)
            z = polynorm(h @ W[pre + "mlp.up"].T, W[pre + "mlp.act"], eps)
            x = x + norm(pre + "norm2b", z @ W[pre + "mlp.down"].T)
        taps.append(x)
    return norm("final.norm", x) @ W["embed"].T, taps


def random_weights(cfg, seed=0, a1_rank=None):
    """Small random weights under the checkpoint's names.  Scales are chosen
    so that activations stay around one and no mechanism is negligible."""
    g = torch.Generator().manual_seed(seed)
    w = {}

    def mat(name, n, k, s=1.0):
        w[name] = (torch.randn(n, k, generator=g) * s / math.sqrt(k))

    def vec(name, n, mean, spread):
        w[name] = mean + spread * torch.randn(n, generator=g)

    def norm(name, n):
        vec(name, n, 1.0, 0.2)
        vec(name + ".b", n, 0.0, 0.1)
        w[name + ".alpha"] = 0.5 + 0.5 * torch.rand((), generator=g)

    width, vocab = cfg["width"], cfg["vocab"]
    w["embed"] = torch.randn(vocab, width, generator=g)
    for i, L in enumerate(cfg["layers"]):
        pre, m = f"l{i}.", L["mixer"]
        H, D, V = m["heads"], m["dim"], m["vdim"]
        for n in ("norm1", "norm1b") + (("norm2", "norm2b")
                                        if L.get("mlp") else ()):
            norm(pre + n, width)
        w[pre + "shift"] = torch.rand(width, generator=g)
        mat(pre + "mix.q", H * D, width)
        if L["type"] == "gla":
            r = a1_rank or 8
            mat(pre + "mix.k", H * D, width)
            mat(pre + "mix.v", H * V, width)
            mat(pre + "mix.g", H * V, width)
            mat(pre + "mix.a1", r, width)
            mat(pre + "mix.a2", H * D, r)
            vec(pre + "mix.a2.b", H * D, 1.0, 1.5)
            vec(pre + "mix.norm", V, 1.0, 0.2)
        else:
            R = m["kv_rank"]
            mat(pre + "mix.dkv", R, width)
            vec(pre + "mix.dkv.norm", R, 1.0, 0.2)
            mat(pre + "mix.uk", H * D, R)
            mat(pre + "mix.uv", H * V, R)
        mat(pre + "mix.o", width, H * V)
        if L.get("mlp"):
            ff = L["mlp"]["ff"]
            mat(pre + "mlp.up", ff, width)
            mat(pre + "mlp.down", width, ff)
            w[pre + "mlp.act"] = torch.tensor([0.8, 0.4, 0.3, 0.1]) \
                + 0.1 * torch.randn(4, generator=g)
    norm("final.norm", width)
    # checkpoints hold bfloat16: round here so both sides read the same
    return {k: t.to(torch.bfloat16) for k, t in w.items()}
