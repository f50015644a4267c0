"""Plain, slow statement of the Kavedra equations, in float64 on the CPU.

One function per mechanism, written query by query and token by token, with
no cache, no batching and nothing imported from the framework.  The tests
compare the framework with this.  Weights are a dict name -> tensor with the
checkpoint's names; the configuration is the plain config.json dict.
"""
import math

import torch

F64 = torch.float64


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm(x, w, eps):
    """The stored weight is the distance from one."""
    return rms(x, eps) * (1.0 + w)


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


# ------------------------------------------------------------------ rotation

def frequencies(rot):
    """Angle per token of every pair, and the factor of cosine and sine."""
    n, base, sc = rot["dims"], rot["base"], rot.get("scaling")
    f = [base ** (-2.0 * i / n) for i in range(n // 2)]
    if not sc:
        return f, 1.0

    def turns(t):
        """The pair that turns t times over the original context."""
        return n * math.log(sc["original"] / (2 * math.pi * t)) \
            / (2 * math.log(base))

    lo = max(math.floor(turns(sc["fast"])), 0)
    hi = min(math.ceil(turns(sc["slow"])), n - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * ramp + fi * (1 - ramp))
    return out, 0.1 * math.log(sc["factor"]) + 1.0


def rotate(x, positions, rot):
    """x [T, ..., dim]; neighbours are a pair, dims past rot's pass."""
    freq, mag = frequencies(rot)
    out = x.clone()
    for t, p in enumerate(positions):
        for i, f in enumerate(freq):
            c, s = mag * math.cos(p * f), mag * math.sin(p * f)
            u, v = x[t, ..., 2 * i], x[t, ..., 2 * i + 1]
            out[t, ..., 2 * i] = u * c - v * s
            out[t, ..., 2 * i + 1] = v * c + u * s
    return out


# -------------------------------------------------------------------- mixers

def softmax_attention(q, k, v, scale, window=None, sink=None, start=0):
    """One head.  q [T, D] are the queries of positions start.., k [N, D] and
    v [N, V] the keys and values of positions 0..  `sink` is one more term of
    the denominator."""
    out = torch.zeros(q.shape[0], v.shape[1], dtype=q.dtype)
    for t in range(q.shape[0]):
        i = start + t
        lo = max(0, i - window + 1) if window else 0
        s = (k[lo:i + 1] @ q[t]) * scale
        top = s.max() if sink is None else torch.maximum(s.max(), sink)
        e = torch.exp(s - top)
        den = e.sum()
        if sink is not None:
            den = den + torch.exp(sink - top)
        out[t] = (e @ v[lo:i + 1]) / den
    return out


def lightning_heads(q, k, v, decay, state=None):
    """q, k [T, H, D], v [T, H, V]; returns (o [T, H, V], last state)."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=q.dtype) if state is None \
        else state.clone()
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for t in range(T):
        for h in range(H):
            S[h] = decay[h] * S[h] + torch.outer(k[t, h], v[t, h])
            out[t, h] = S[h].T @ q[t, h]
    return out, S


def gated_norm(o, w, gate, eps):
    """All heads of a token normed together."""
    return rms(o, eps) * w * sigmoid(gate)


def lightning_mixer(h, p, m, eps):
    H, D, V = m["heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q = silu(h @ p("q").T).view(T, H, D)
    k = silu(h @ p("k").T).view(T, H, D)
    v = silu(h @ p("v").T).view(T, H, V)
    o, _ = lightning_heads(q, k, v, m["decay"])
    return gated_norm(o.reshape(T, H * V), p("norm"), h @ p("g").T, eps) \
        @ p("o").T


def attention_mixer(h, p, m, eps):
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    pos = range(T)
    q = rotate((h @ p("q").T + p("q.b")).view(T, H, D), pos, m["rot"])
    k = rotate((h @ p("k").T + p("k.b")).view(T, G, D), pos, m["rot"])
    v = (h @ p("v").T + p("v.b")).view(T, G, V)
    sink = p("sink")
    return torch.cat([softmax_attention(
        q[:, i], k[:, i // (H // G)], v[:, i // (H // G)], m["scale"],
        sink=sink[i]) for i in range(H)], -1) @ p("o").T


def latent_heads(q, c, kr, uk, uv, scale, window, start=0):
    """q [T, H, D + Dr], c [N, R], kr [N, Dr]; uk [H, D, R], uv [H, V, R]."""
    heads = []
    for i in range(uk.shape[0]):
        k = torch.cat([c @ uk[i].T, kr], -1)
        heads.append(softmax_attention(q[:, i], k, c @ uv[i].T, scale,
                                       window, start=start))
    return torch.cat(heads, -1)


def latent_mixer(h, p, m, eps):
    H, D, V, R, Dr = (m[n] for n in ("heads", "dim", "vdim", "kv_rank",
                                     "rot_dim"))
    T = h.shape[0]
    q = (h @ p("q").T).view(T, H, D + Dr)
    q = torch.cat([q[..., :D], rotate(q[..., D:], range(T), m["rot"])], -1)
    d = h @ p("dkv").T
    c = rms(d[:, :R], eps) * p("dkv.norm")
    kr = rotate(d[:, R:], range(T), m["rot"])
    window = m["mask"]["size"] if m.get("mask") else None
    o = latent_heads(q, c, kr, p("uk").view(H, D, R), p("uv").view(H, V, R),
                     m["scale"], window)
    return (o * sigmoid(h @ p("g").T)) @ p("o").T


MIXERS = {"lightning": lightning_mixer, "attention": attention_mixer,
          "latent_attention": latent_mixer}


# --------------------------------------------------------------------- model

def dense_ff(h, p):
    return (silu(h @ p("gate").T) * (h @ p("up").T)) @ p("down").T


def enter_pass(x, x0, w_in, step):
    return torch.cat([x, x0], -1) @ w_in.T + step


def run(cfg, weights, tokens):
    """Logits [T, vocab] of a whole sequence, and the residual stream after
    every layer run."""
    eps = cfg["norm"]["eps"]
    w = {n: t.to(F64) for n, t in weights.items()}
    x = x0 = w["embed"][torch.as_tensor(tokens)]
    n = len(cfg["layers"])
    lp = cfg.get("loop") or {"start": n, "stop": n, "times": 0}
    order = [(i, None) for i in range(lp["start"])]
    for t in range(lp["times"]):
        order += [(i, t if i == lp["start"] else None)
                  for i in range(lp["start"], lp["stop"])]
    order += [(i, None) for i in range(lp["stop"], n)]
    layers = []
    for i, entering in order:
        layer, pre = cfg["layers"][i], f"l{i}."
        if entering is not None:
            x = enter_pass(x, x0, w["loop.in"], w["loop.step"][entering])
        x = x + MIXERS[layer["type"]](
            norm(x, w[pre + "norm1"], eps), lambda k: w[pre + "mix." + k],
            layer["mixer"], eps)
        if layer["mlp"]:
            x = x + dense_ff(norm(x, w[pre + "norm2"], eps),
                             lambda k: w[pre + "mlp." + k])
        layers.append(x)
    logits = norm(x, w["final.norm"], eps) @ w["head"].T * cfg["logit_scale"]
    return logits, torch.stack(layers)


def random_weights(cfg, seed=0):
    """bf16 weights with the checkpoint's names and shapes."""
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]
    out = {}

    def mat(name, n, k, s=1.0):
        out[name] = (torch.randn(n, k, generator=g) * s / math.sqrt(k)) \
            .to(torch.bfloat16)

    def vec(name, n, mean=0.0, spread=0.2):
        out[name] = (mean + spread * torch.randn(n, generator=g)) \
            .to(torch.bfloat16)

    out["embed"] = torch.randn(cfg["vocab"], W, generator=g) \
        .to(torch.bfloat16)
    if cfg.get("loop"):
        mat("loop.in", W, 2 * W)
        out["loop.step"] = (0.3 * torch.randn(cfg["loop"]["times"], W,
                                              generator=g)) \
            .to(torch.bfloat16)
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        x = p + "mix."
        H, D, V = m["heads"], m["dim"], m["vdim"]
        vec(p + "norm1", W)
        if layer["type"] == "lightning":
            mat(x + "q", H * D, W)
            mat(x + "k", H * D, W)
            mat(x + "v", H * V, W)
            mat(x + "g", H * V, W)
            vec(x + "norm", H * V, 1.0)
        elif layer["type"] == "attention":
            G = m["kv_heads"]
            for n, rows in (("q", H * D), ("k", G * D), ("v", G * V)):
                mat(x + n, rows, W, 1.5)
                vec(x + n + ".b", rows, 0.0, 0.5)
            vec(x + "sink", H, 0.5, 1.0)
        else:
            R, Dr = m["kv_rank"], m["rot_dim"]
            mat(x + "q", H * (D + Dr), W, 1.5)
            mat(x + "dkv", R + Dr, W)
            vec(x + "dkv.norm", R, 1.0)
            mat(x + "uk", H * D, R)
            mat(x + "uv", H * V, R)
            mat(x + "g", H * V, W)
        mat(x + "o", W, H * V)
        if layer["mlp"]:
            vec(p + "norm2", W)
            F = layer["mlp"]["ff"]
            mat(p + "mlp.gate", F, W)
            mat(p + "mlp.up", F, W)
            mat(p + "mlp.down", W, F)
    vec("final.norm", W)
    mat("head", cfg["vocab"], W)
    return out
