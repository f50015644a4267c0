"""Plain, slow statement of the Pemidra equations, in float64 on the CPU.

One function per mechanism, written token by token and key by key, with no
cache, no batching and nothing imported from the framework.  The tests
compare the framework with this.  Weights are a dict name -> tensor with the
checkpoint's names; the configuration is the plain config.json dict.
"""
import math

import torch

F64 = torch.float64
UNIT_EPS = 1e-6                  # inside the root of a unit vector


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + UNIT_EPS)


def layer_norm(x, w, b, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w + b


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return torch.where(z > 30.0, z, torch.log1p(torch.exp(z.clamp(max=30.0))))


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi)
                                     * (z + 0.044715 * z ** 3)))


# ------------------------------------------------------------ softmax mixer

def rotate(x, positions, rot):
    """x [T, ..., dim]; dimension i turns with dimension i + dims / 2."""
    half, base = rot["dims"] // 2, rot["base"]
    out = x.clone()
    for t, p in enumerate(positions):
        for i in range(half):
            a = p * base ** (-2.0 * i / rot["dims"])
            u, v = x[t, ..., i], x[t, ..., i + half]
            out[t, ..., i] = u * math.cos(a) - v * math.sin(a)
            out[t, ..., i + half] = v * math.cos(a) + u * math.sin(a)
    return out


def chunk_attention(q, k, v, scale, size, start=0, sink=True):
    """One head.  q [T, D] are the queries of positions start.., k [N, D] and
    v [N, V] belong to positions 0..; a query sees the keys of its own chunk
    of `size` positions.  The denominator has one added."""
    out = torch.zeros(q.shape[0], v.shape[1], dtype=q.dtype)
    for t in range(q.shape[0]):
        i = start + t
        lo = i // size * size if size else 0
        s = (k[lo:i + 1] @ q[t]) * scale
        top = s.max().clamp(min=0.0) if sink else s.max()
        e = torch.exp(s - top)
        out[t] = (e @ v[lo:i + 1]) / (e.sum()
                                      + (torch.exp(-top) if sink else 0.0))
    return out


def attention_mixer(h, p, m, eps):
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q = rms((h @ p("q").T).view(T, H, D), eps) * p("q.norm")
    k = rms((h @ p("k").T).view(T, G, D), eps) * p("k.norm")
    v = rms((h @ p("v").T).view(T, G, V), eps)
    q, k = rotate(q, range(T), m["rot"]), rotate(k, range(T), m["rot"])
    gate, temp = sigmoid(h @ p("g").T), p("temp")
    return torch.cat([chunk_attention(
        q[:, i], k[:, i // (H // G)], v[:, i // (H // G)],
        m["scale"] * temp[i], m["mask"]["size"]) * gate[:, i:i + 1]
        for i in range(H)], -1) @ p("o").T


# -------------------------------------------------------- recurrent mixers

def retention_heads(q, k, v, decay, state=None):
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


def retention_mixer(h, p, m, eps):
    H, D, V = m["heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q = (h @ p("q").T).view(T, H, D)
    k = (h @ p("k").T).view(T, H, D) * D ** -0.5
    v = (h @ p("v").T).view(T, H, V)
    o, _ = retention_heads(q, k, v, m["decay"])
    return (rms(o, eps).reshape(T, H * V) * silu(h @ p("g").T)) @ p("o").T


def short_conv(x, w, before=None):
    """x [T, C], w [C, taps] with the current token's weight last; `before`
    [taps - 1, C] are the inputs ahead of x, none at a sequence's start."""
    T, C = x.shape
    taps = w.shape[1]
    if before is None:
        before = torch.zeros(taps - 1, C, dtype=x.dtype)
    row = torch.cat([before, x])
    out = torch.zeros_like(x)
    for t in range(T):
        for j in range(taps):
            out[t] += w[:, j] * row[t + j]
    return out


def gated_delta_heads(q, k, v, g, beta, state=None):
    """q, k, g [T, H, D], v [T, H, V], beta [T, H]; g and beta are the
    factors themselves."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=q.dtype) if state is None \
        else state.clone()
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for t in range(T):
        for h in range(H):
            S[h] = g[t, h][:, None] * S[h]
            u = beta[t, h] * (v[t, h] - S[h].T @ k[t, h])
            S[h] = S[h] + torch.outer(k[t, h], u)
            out[t, h] = S[h].T @ q[t, h]
    return out, S


def gated_delta_mixer(h, p, m, eps):
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T, R = h.shape[0], m["heads"] // m["kv_heads"]
    conv = lambda n: silu(short_conv(h @ p(n).T, p(n + ".conv")))
    q = unit(conv("q").view(T, G, D)) * D ** -0.5
    k = unit(conv("k").view(T, G, D))
    v = conv("v").view(T, H, V)
    z = (h @ p("a1").T) @ p("a2").T + p("dt_bias")
    g = torch.exp(-torch.exp(p("A_log"))[None, :, None]
                  * softplus(z).view(T, H, D))
    q, k = q.repeat_interleave(R, 1), k.repeat_interleave(R, 1)
    o, _ = gated_delta_heads(q, k, v, g, sigmoid(h @ p("b").T))
    gate = sigmoid((h @ p("g1").T) @ p("g2").T)
    return ((rms(o, eps) * p("norm")).reshape(T, H * V) * gate) @ p("o").T


def parallel_mixer(h, p, m, eps):
    left = attention_mixer(h, lambda n: p("left." + n), m["left"], eps)
    right = gated_delta_mixer(h, lambda n: p("right." + n), m["right"], eps)
    return 0.5 * (rms(left, eps) * p("left.out")
                  + rms(right, eps) * p("right.out"))


def general_delta_heads(r, k, v, w, a, state=None):
    """All [T, H, D]; w and a are the factors themselves."""
    T, H, D = r.shape
    S = torch.zeros(H, D, D, dtype=r.dtype) if state is None \
        else state.clone()
    out = torch.zeros(T, H, D, dtype=r.dtype)
    for t in range(T):
        for h in range(H):
            u = unit(k[t, h])
            S[h] = w[t, h][:, None] * S[h] \
                - torch.outer(a[t, h] * u, S[h].T @ u) \
                + torch.outer(k[t, h], v[t, h])
            out[t, h] = S[h].T @ r[t, h]
    return out, S


def general_delta_mixer(h, p, m, eps):
    H, D = m["heads"], m["dim"]
    T = h.shape[0]
    r, k, v = ((h @ p(n).T).view(T, H, D) for n in "rkv")
    z = torch.tanh(h @ p("w1").T) @ p("w2").T + p("w0")
    w = torch.exp(-math.exp(-0.5) * sigmoid(z)).view(T, H, D)
    a = sigmoid(h @ p("a").T + p("a.b")).view(T, H, D)
    o, _ = general_delta_heads(r, k, v, w, a)
    return (rms(o, eps).reshape(T, H * D) * p("norm")
            * sigmoid(h @ p("g").T)) @ p("o").T


MIXERS = {"retention": retention_mixer, "parallel": parallel_mixer,
          "general_delta": general_delta_mixer}


# --------------------------------------------------------------------- model

def dense_ff(h, p):
    return (gelu_tanh(h @ p("gate").T) * (h @ p("up").T)) @ p("down").T


def run(cfg, weights, tokens):
    """Logits [T, vocab] of a whole sequence, and the residual stream after
    every layer."""
    eps, alpha = cfg["norm"]["eps"], cfg["postln_alpha"]
    w = {n: t.to(F64) for n, t in weights.items()}
    x = w["embed"][torch.as_tensor(tokens)]
    layers = []
    for i, layer in enumerate(cfg["layers"]):
        pre = f"l{i}."
        norm = lambda n, z: layer_norm(z, w[pre + n], w[pre + n + ".b"], eps)
        y = MIXERS[layer["type"]](x, lambda k: w[pre + "mix." + k],
                                  layer["mixer"], eps)
        x = norm("norm1", alpha * x + w[pre + "ls1"] * y)
        if layer["mlp"]:
            y = dense_ff(x, lambda k: w[pre + "mlp." + k])
            x = norm("norm2", alpha * x + w[pre + "ls2"] * y)
        layers.append(x)
    logits = layer_norm(x, w["final.norm"], w["final.norm.b"], eps) \
        @ w["head"].T
    return logits, torch.stack(layers)


def random_weights(cfg, seed=0, ranks=(6, 13, 9)):
    """bf16 weights with the checkpoint's names and shapes; ranks of the
    gated rule's decays and gates and of the generalized rule's decays."""
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]
    out = {}

    def mat(name, n, k=W, s=1.0):
        out[name] = (torch.randn(n, k, generator=g) * s / math.sqrt(k)) \
            .to(torch.bfloat16)

    def vec(name, n, mean=0.0, spread=0.2):
        out[name] = (mean + spread * torch.randn(n, generator=g)) \
            .to(torch.bfloat16)

    def norm(name):
        vec(name, W, 1.0)
        vec(name + ".b", W)

    def attention(x, m):
        H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        mat(x + "q", H * D)
        mat(x + "k", G * D)
        mat(x + "v", G * V)
        vec(x + "q.norm", D, 1.3)
        vec(x + "k.norm", D, 1.3)
        vec(x + "temp", H, 1.0, 0.4)
        mat(x + "g", H, s=2.0)
        mat(x + "o", W, H * V)

    def gated_delta(x, m):
        H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        for n, rows in (("q", G * D), ("k", G * D), ("v", H * V)):
            mat(x + n, rows)
            mat(f"{x}{n}.conv", rows, m["conv"], 1.5)
        mat(x + "b", H)
        vec(x + "A_log", H, 0.0, 1.0)
        vec(x + "norm", V, 1.0)
        mat(x + "a1", ranks[0])
        mat(x + "a2", H * D, ranks[0])
        vec(x + "dt_bias", H * D, -2.0, 1.5)
        mat(x + "g1", ranks[1])
        mat(x + "g2", H * V, ranks[1])
        mat(x + "o", W, H * V)

    out["embed"] = torch.randn(cfg["vocab"], W, generator=g) \
        .to(torch.bfloat16)
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        x = p + "mix."
        norm(p + "norm1")
        vec(p + "ls1", W, 1.0)
        if layer["type"] == "retention":
            H, D, V = m["heads"], m["dim"], m["vdim"]
            mat(x + "q", H * D)
            mat(x + "k", H * D)
            mat(x + "v", H * V)
            mat(x + "g", H * V)
            mat(x + "o", W, H * V)
        elif layer["type"] == "general_delta":
            n = m["heads"] * m["dim"]
            for c in "rkvga":
                mat(x + c, n)
            vec(x + "a.b", n)
            mat(x + "w1", ranks[2])
            mat(x + "w2", n, ranks[2], 2.0)
            vec(x + "w0", n, -1.0, 1.5)
            vec(x + "norm", n, 1.0)
            mat(x + "o", W, n)
        else:
            attention(x + "left.", m["left"])
            gated_delta(x + "right.", m["right"])
            vec(x + "left.out", W, 1.0)
            vec(x + "right.out", W, 1.0)
        if layer["mlp"]:
            norm(p + "norm2")
            vec(p + "ls2", W, 1.0)
            F = layer["mlp"]["ff"]
            mat(p + "mlp.gate", F)
            mat(p + "mlp.up", F)
            mat(p + "mlp.down", W, F)
    norm("final.norm")
    mat("head", cfg["vocab"])
    return out
