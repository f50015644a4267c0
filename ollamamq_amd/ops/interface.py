"""Op dispatch: hand-written gfx950 HIP kernels on GPU, fp32 torch on CPU.

Policy (task requirement): on a GPU box the HIP extension MUST be present —
ops fail loudly rather than falling back to eager PyTorch, so a passing GPU
test is evidence the native path ran.  Set OLLAMAMQ_FORCE_REF=1 to force the
reference path explicitly (used only by numerics tests to produce oracles).
"""
from __future__ import annotations

import os
from dataclasses import dataclass
from typing import List, NamedTuple, Optional, Union

import torch

from . import reference as ref


def _use_hip(t: torch.Tensor) -> bool:
    if not t.is_cuda:
        return False
    if os.environ.get("OLLAMAMQ_FORCE_REF") == "1":
        return False
    from . import hip  # deferred: imports/builds the extension
    hip.require()      # raises if the extension is missing on a GPU box
    return True


@dataclass
class AttnMeta:
    """Per-forward attention metadata (flat varlen layout).

    mode: "prefill" (multi-token queries), "decode" (1 token/seq) or
    "mixed" (the first n_decode sequences are single-token decodes, the
    rest are prefill chunks — one forward shares the weight pass).
    slot_ids : [S] int32  kv-cache slot of each sequence in batch order
    seq_lens : [S] int32  total KV length per slot AFTER the kv_append
    cu_q     : [S+1] int32 exclusive prefix sum of per-seq query counts
    logits_idx: [S] int64 flat indices of each sequence's last token
                (None = all tokens get logits)
    """
    mode: str
    slot_ids: torch.Tensor
    seq_lens: torch.Tensor
    cu_q: torch.Tensor
    logits_idx: Optional[torch.Tensor]
    max_q: int
    max_kv: int
    n_decode: int = 0
    # sliding-window attention (Mistral-style): query at position p attends
    # keys [max(0, p - window + 1), p]; 0 = full causal
    window: int = 0
    # host copies of the batch layout (None in a captured decode step):
    # tokens per sequence and cached length per sequence
    q_lens: Optional[List[int]] = None
    kv_lens: Optional[List[int]] = None
    slots: Optional[List[int]] = None

    @property
    def one_each(self) -> bool:
        """Every sequence brings exactly one token."""
        return self.mode == "decode"

    @property
    def n_single(self) -> int:
        """Leading rows that are single tokens of their sequence."""
        return (self.slot_ids.shape[0] if self.one_each
                else self.n_decode if self.mode == "mixed" else 0)

    def layout(self):
        """(slots, tokens per sequence, cached lengths) as host lists."""
        if self.q_lens is None:
            cu = self.cu_q.tolist()
            self.q_lens = [b - a for a, b in zip(cu, cu[1:])]
            self.kv_lens = self.seq_lens.tolist()
            self.slots = self.slot_ids.tolist()
        return self.slots, self.q_lens, self.kv_lens


class DyT(NamedTuple):
    """Dynamic tanh: tanh(alpha * x) * w + b (w, b fp32)."""
    w: torch.Tensor
    b: torch.Tensor
    alpha: float


class TokenShift(NamedTuple):
    """h[t] + (h[t-1] - h[t]) * mix; `prev` [slots, W] fp32 keeps every
    sequence's last h between steps (zero at position 0)."""
    mix: torch.Tensor
    prev: torch.Tensor
    slot_ids: torch.Tensor        # per token
    positions: torch.Tensor       # per token
    meta: AttnMeta


class Partials(NamedTuple):
    """A matrix product as [parts, rows, cols] fp32 partial sums; the
    consumer folds them."""
    parts: torch.Tensor


class Weighted(NamedTuple):
    """A row as a weighted sum of several: sum_s share[r, s] * parts[r, s];
    parts [rows, n, cols] bf16 or fp32, share [rows, n] fp32.  The consumer
    adds them up."""
    parts: torch.Tensor
    share: torch.Tensor


class FragRows(NamedTuple):
    """A bf16 activation [rows, cols] in the layout in which the
    weight-streaming product reads it (GPU decode, up to 64 rows)."""
    buf: torch.Tensor
    rows: int
    cols: int


class Columns(NamedTuple):
    """Columns of a fused projection from `first` on, as many as the consumer
    needs; the projection may be Partials."""
    p: object
    first: int


class Rope(NamedTuple):
    """Rotary positions: table [positions, dims] fp32 holds (cos, sin) of
    every pair of a head's first `dims` dimensions: (2i, 2i+1), or
    (i, i + dims/2) with `halves`."""
    table: torch.Tensor
    dims: int
    halves: bool = False


class LayerNorm(NamedTuple):
    """(x - mean) / sqrt(variance + eps) * w + b (w, b fp32)."""
    w: torch.Tensor
    b: torch.Tensor


class Branches(NamedTuple):
    """Results of sublayers side by side: share * sum N(y) * w over the
    (y, w) pairs, N the division by a row's root mean square.  The consumer
    norms them and adds them up."""
    pairs: tuple
    share: float


class LatentWeights(NamedTuple):
    """k = uk c, v = uv c per head; uk [H, D, R], uk_t [H, R, D] and
    uv [H, V, R] are views or copies of the same values.  With rot_dim, query
    heads are [D, rot_dim] and the cached row ends in a key part of that
    width which all heads share.  A query sees `window` tokens, itself
    included (0: all before it)."""
    uk: torch.Tensor
    uk_t: torch.Tensor
    uv: torch.Tensor
    scale: float
    rot_dim: int = 0
    window: int = 0


class SoftmaxAttn(NamedTuple):
    """Softmax attention over paged keys and values; `sink` (fp32 per query
    head, or None) is one more logit of the denominator.  A query sees
    `window` tokens, itself included (0: all before it), or, with `chunk`,
    the tokens of its own chunk of that many positions."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    sink: Optional[torch.Tensor] = None
    window: int = 0
    chunk: int = 0

    def reach(self, kv: int) -> int:
        """Most keys that a query of a context of kv tokens sees."""
        return min(kv, self.window or self.chunk or kv)


class HeadNorms(NamedTuple):
    """What happens to each head of a projection before attention: RMS norm
    with weights of the head's width (q, k, fp32), of the values without a
    weight, and a factor per query head (fp32, or None)."""
    q: torch.Tensor
    k: torch.Tensor
    values: bool
    gain: Optional[torch.Tensor]
    eps: float


LIGHTNING_CHUNK = 64


def decay_powers(decay, device) -> torch.Tensor:
    """fp32 [heads, LIGHTNING_CHUNK + 1]: powers of every head's decay."""
    steps = torch.arange(LIGHTNING_CHUNK + 1, dtype=torch.float64)
    d = torch.tensor(decay, dtype=torch.float64)
    return (d[:, None] ** steps).float().to(device).contiguous()


class LightningWeights(NamedTuple):
    """Columns of the fused projection, and what the recurrence, the norm and
    the output gate read."""
    heads: int
    dim: int
    vdim: int
    offsets: tuple                # columns of q, k, v, gate
    powers: torch.Tensor          # decay_powers
    norm: Optional[torch.Tensor]  # fp32 [heads * vdim], None: no weight
    eps: float
    act: bool = True              # silu of q, k and v
    scale: float = 1.0            # of the results
    per_head: bool = False        # norm of every head, not of all together
    gate: str = "sigmoid"         # or "silu"


UNIT_EPS = 1e-6       # inside the root of a unit vector


class LowRank(NamedTuple):
    """The second matrix [N, rank] of a low-rank projection and, on the GPU,
    its copy in the order in which the matrix cores take it."""
    w: torch.Tensor
    packed: Optional[torch.Tensor] = None

    @property
    def rank(self) -> int:
        return self.w.shape[1]


def low_rank(w: torch.Tensor) -> LowRank:
    if not w.is_cuda:
        return LowRank(w)
    from . import hip
    return LowRank(w, hip.pack_operand(w))


class GatedDeltaWeights(NamedTuple):
    """Gated delta rule with a decay per key channel.  Columns of the fused
    projection (q, k and v follow one another), the short convolution over
    them, the low-rank projections of decays and output gate."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    offsets: tuple                # columns of q|k|v, beta, decay, gate
    conv: torch.Tensor            # fp32 [taps, channels], the current last
    a2: LowRank                   # [heads * dim, rank]
    rate: torch.Tensor            # fp32 [heads], exp of the stored logarithm
    dt_bias: torch.Tensor         # fp32 [heads * dim]
    g2: LowRank                   # [heads * vdim, rank]
    norm: torch.Tensor            # fp32 [vdim]
    eps: float


class GeneralDeltaWeights(NamedTuple):
    """Generalized delta rule: decay and removal rate per key channel.
    Columns of the fused projection and the decays' low-rank projection,
    whose columns and rank are whole vectors of 8."""
    heads: int
    dim: int
    offsets: tuple                # columns of r, k, v, removal, gate, decay
    w2: LowRank                   # [heads * dim, rank]
    w0: torch.Tensor              # fp32 [heads * dim]
    a_bias: torch.Tensor          # fp32 [heads * dim]
    norm: torch.Tensor            # fp32 [heads * dim]
    eps: float


class GlaWeights(NamedTuple):
    """Columns of the fused projection, and what the recurrence reads."""
    heads: int
    dim: int
    vdim: int
    rank: int
    offsets: tuple                # columns of q, k, v, gate, low rank
    a2: torch.Tensor              # [heads * dim, rank]
    a2_b: torch.Tensor            # fp32
    norm: torch.Tensor            # fp32 [vdim]
    tau: float
    eps: float


class SigmoidAttn(NamedTuple):
    """Attention whose weight for a key `dist` tokens back is
    sigmoid(cap(scale * q.k) - decay * ln(1 + reach * dist) + bias), with
    cap(s) = softcap * tanh(s / softcap) (softcap 0: none); decay, reach and
    bias are fp32 per query head.  A query sees `window` tokens, itself
    included (0: all before it)."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: float
    decay: torch.Tensor
    reach: torch.Tensor
    bias: torch.Tensor
    window: int


MOE_BLOCK = 16     # gate and up rows alternate in blocks of this many


class MoeWeights(NamedTuple):
    """Experts of silu(gate x) * (up x) -> down.  gate_up [E, 2*F, K] holds
    16 gate rows, then their 16 up rows, and so on, so that a tile of the
    product has both; F is the experts' width filled up with zeros to
    whole tiles.  down [E, N, F]."""
    router: torch.Tensor          # [E, K]
    gate_up: torch.Tensor
    down: torch.Tensor
    top: int


def moe_weights(router, experts, top, put) -> MoeWeights:
    """`experts`: (gate [F, K], up [F, K], down [N, F]) each; put moves a
    tensor to where and how the model keeps its weights."""
    F, K = experts[0][0].shape
    N = experts[0][2].shape[0]
    pad = -(-F // 64) * 64
    E, b = len(experts), MOE_BLOCK
    gu = down = None
    for e, (gate, up, dn) in enumerate(experts):
        gate, up, dn = put(gate), put(up), put(dn)
        if gu is None:
            gu = gate.new_zeros(E, pad, 2, K)
            down = dn.new_zeros(E, N, pad)
        gu[e, :F, 0], gu[e, :F, 1] = gate, up
        down[e, :, :F] = dn
    gu = gu.view(E, pad // b, b, 2, K).transpose(2, 3).reshape(E, 2 * pad, K)
    return MoeWeights(router, gu.contiguous(), down, top)


def embedding(tokens: torch.Tensor, table: torch.Tensor) -> torch.Tensor:
    if _use_hip(table):
        from . import hip
        return hip.embedding(tokens, table)
    return table.index_select(0, tokens.long())


def rmsnorm_residual(x, residual, weight, eps):
    if _use_hip(x):
        from . import hip
        return hip.rmsnorm_residual(x, residual, weight, eps)
    return ref.rmsnorm_residual(x, residual, weight, eps)


def rope(q, k, positions, cos, sin):
    if _use_hip(q):
        from . import hip
        return hip.rope(q, k, positions, cos, sin)
    return ref.rope(q, k, positions, cos, sin)


def rope_append(cache, layer, q, k, v, positions, slot_ids, cos, sin):
    """Fused RoPE + KV append (one pass); falls back to the two reference
    ops on CPU."""
    if _use_hip(q):
        from . import hip
        return hip.rope_append(cache, layer, q, k, v, positions, slot_ids,
                               cos, sin)
    ref.rope(q, k, positions, cos, sin)
    ref.kv_append(cache, layer, k, v, slot_ids, positions)


def kv_append(cache, layer, k, v, slot_ids, positions):
    if _use_hip(k):
        from . import hip
        return hip.kv_append(cache, layer, k, v, slot_ids, positions)
    return ref.kv_append(cache, layer, k, v, slot_ids, positions)


def attention(q, cache, layer, meta: AttnMeta):
    if _use_hip(q):
        from . import hip
        if meta.mode == "decode":
            return hip.attention_decode(q, cache, layer, meta)
        if meta.mode == "mixed":
            return hip.attention_mixed(q, cache, layer, meta)
        return hip.attention_prefill(q, cache, layer, meta)
    # the fp32 reference handles any varlen layout uniformly
    return ref.attention(q, cache, layer, meta)


def linear(x, weight, bias=None, packed=None):
    """y = x @ weight.T (+ bias).  Library GEMM for prefill shapes; on the
    decode path (M<=64) a hand-written weight-streaming MFMA kernel runs
    over the pre-packed copy when `packed` is provided (hipBLASLt measured
    1.8-4.6 TB/s vs the ~6.3 TB/s streaming roofline on these shapes)."""
    if _use_hip(weight):
        from . import hip
        return hip.linear(x, weight, bias, packed)
    return torch.nn.functional.linear(x, weight, bias)


def pack_weight(w):
    """MFMA-fragment-order packed copy for the decode GEMM (GPU only).
    Every projection is packed: the fused decode chain streams all of
    them (the per-shape lib-vs-stream policy only applies to the generic
    non-chain dispatch in hip.linear)."""
    if w.is_cuda:
        from . import hip
        if hip.available():
            return hip.pack_weight(w)
    return None


def linear_parts(x, weight, packed=None,
                 most=8) -> Union[torch.Tensor, Partials]:
    """As linear, but a split product may come back as its partial sums, at
    most `most` of them (few where several consumers add them up)."""
    if _use_hip(weight):
        from . import hip
        return hip.linear_parts(x, weight, packed, most)
    return torch.nn.functional.linear(x, weight)


def dyt_residual(x, y, post: Optional[DyT], pre: DyT,
                 shift: Optional[TokenShift] = None, embed=None, tokens=None,
                 rows=None, need_x=True, frag=False):
    """One pass between two matrix products: x' = x + post(y), h = pre(x'),
    then the token shift.  x is fp32 [T, W], or None for the embedding rows
    of `tokens`; y a tensor, Partials or None; `rows` selects the rows to
    compute; frag returns h as FragRows.  Returns (x', h)."""
    if _use_hip(pre.w):
        from . import hip
        return hip.dyt_residual(x, y, post, pre, shift, embed, tokens, rows,
                                need_x, frag)
    return ref.dyt_residual(x, y, post, pre, shift, embed, tokens, rows)


def linear_f32(x, weight, packed=None) -> Union[torch.Tensor, Partials]:
    """As linear_parts, the result fp32 whatever the operands' type."""
    if _use_hip(weight):
        from . import hip
        return hip.linear_f32(x, weight, packed)
    return torch.nn.functional.linear(x.float(), weight.float())


def polynorm(z, coef, eps, frag=False):
    """a N(z) + b N(z^2) + c N(z^3) + e with coef = (a, b, c, e) and N the
    division by the row's root mean square."""
    t = z.parts if isinstance(z, Partials) else z
    if _use_hip(t):
        from . import hip
        return hip.polynorm(z, coef, eps, frag)
    return ref.polynorm(z, coef, eps)


def latent_append(cache, run, d, weight, slot_ids, positions, eps):
    """RMS norm of d [T, R] and append to the run's paged latent pool."""
    if _use_hip(d):
        from . import hip
        return hip.latent_append(cache, run, d, weight, slot_ids, positions,
                                 eps)
    return ref.latent_append(cache, run, d, weight, slot_ids, positions, eps)


def latent_rope_append(p, cache, run, w: LatentWeights, norm, eps,
                       rope: Rope, slot_ids, positions):
    """Split the projection p (columns q [H, D + rot_dim] | latent | shared
    key part; a tensor or Partials), rotate, norm the latent, append latent
    and key part to the run's pool.  -> queries [T, H * (D + rot_dim)]."""
    t = p.parts if isinstance(p, Partials) else p
    if _use_hip(t):
        from . import hip
        return hip.latent_rope_append(p, cache, run, w, norm, eps, rope,
                                      slot_ids, positions)
    return ref.latent_rope_append(p, cache, run, w, norm, eps, rope,
                                  slot_ids, positions)


def latent_attention(q, cache, run, w: LatentWeights, slot_ids, positions,
                     meta: AttnMeta, frag=False,
                     gate: Optional[Columns] = None):
    """Causal softmax attention whose keys and values are linear in the
    cached latent.  q [T, H*(D+rot_dim)] (rows may be strided) -> [T, H*V],
    times the sigmoid of the gate's columns."""
    if _use_hip(q):
        from . import hip
        return hip.latent_attention(q, cache, run, w, slot_ids, positions,
                                    meta, frag, gate)
    return ref.latent_attention(q, cache, run, w, meta, gate)


def rope_qkv_append(p, bias, cache, run, w: SoftmaxAttn, rope: Rope,
                    slot_ids, positions):
    """Split the projection p (columns q | k | v; a tensor or Partials), add
    its bias (fp32, or None), rotate queries and keys, append keys and values
    to the run's paged pools.  -> queries [T, H, D'], rows filled up with
    zeros as the pool's are."""
    t = p.parts if isinstance(p, Partials) else p
    if _use_hip(t):
        from . import hip
        return hip.rope_qkv_append(p, bias, cache, run, w, rope, slot_ids,
                                   positions)
    return ref.rope_qkv_append(p, bias, cache, run, w, rope, slot_ids,
                               positions)


def qkv_norm_rope_append(p, norms: HeadNorms, cache, run, w: SoftmaxAttn,
                         rope: Rope, slot_ids, positions):
    """Split the projection p (columns q | k | v; a tensor or Partials), norm
    every head, rotate queries and keys, append keys and values to the run's
    paged pools.  -> queries [T, H, D'], rows filled up with zeros as the
    pool's are."""
    t = p.parts if isinstance(p, Partials) else p
    if _use_hip(t):
        from . import hip
        return hip.qkv_norm_rope_append(p, norms, cache, run, w, rope,
                                        slot_ids, positions)
    return ref.qkv_norm_rope_append(p, norms, cache, run, w, rope, slot_ids,
                                    positions)


def softmax_attention(q, cache, run, w: SoftmaxAttn, slot_ids, positions,
                      meta: AttnMeta, frag=False,
                      gate: Optional[Columns] = None):
    """Causal softmax attention over the run's paged keys and values; q as
    rope_qkv_append returns it.  -> [T, H*V], a head's result times the
    sigmoid of its gate column."""
    if _use_hip(q):
        from . import hip
        return hip.softmax_attention(q, cache, run, w, slot_ids, positions,
                                     meta, frag, gate)
    return ref.softmax_attention(q, cache, run, w, meta, gate)


def lightning(p, w: LightningWeights, state, slot_ids, positions,
              meta: AttnMeta, frag=False):
    """Linear attention with one decay per head over the fused projection
    p [T, ...] (a tensor or Partials); state [slots, H, D, V] fp32 is read
    and advanced.  Norm and output gate included.  -> [T, H*V]."""
    if _use_hip(w.powers):
        from . import hip
        return hip.lightning(p, w, state, slot_ids, positions, meta, frag)
    return ref.lightning(p, w, state, meta)


def gla(p, w: GlaWeights, state, slot_ids, positions, meta: AttnMeta,
        frag=False):
    """Gated linear attention over the fused projection p [T, ...]; state
    [slots, H, D, V] fp32 is read and advanced.  Head norm and output gate
    included.  -> [T, H*V]."""
    if _use_hip(p):
        from . import hip
        return hip.gla(p, w, state, slot_ids, positions, meta, frag)
    return ref.gla(p, w, state, meta)


def gated_delta(p, w: GatedDeltaWeights, state, conv_state, slot_ids,
                positions, meta: AttnMeta, frag=False):
    """Gated delta rule over the fused projection p [T, ...] (a tensor or
    Partials):
        S <- diag(g) S,  S <- S + k (beta (v - S^T k))^T,  o = S^T q.
    state [slots, H, D, V] and conv_state [slots, taps - 1, channels], both
    fp32, are read and advanced.  Head norm and output gate included.
    -> [T, H*V]."""
    if _use_hip(w.norm):
        from . import hip
        return hip.gated_delta(p, w, state, conv_state, slot_ids, positions,
                               meta, frag)
    return ref.gated_delta(p, w, state, conv_state, meta)


def general_delta(p, w: GeneralDeltaWeights, state, slot_ids, positions,
                  meta: AttnMeta, frag=False):
    """Generalized delta rule over the fused projection p [T, ...] (a tensor
    or Partials), u the unit key:
        S <- diag(w) S - (a * u) (S^T u)^T + k v^T,  o = S^T r.
    state [slots, H, D, D] fp32 is read and advanced.  Head norm and output
    gate included.  -> [T, H*D]."""
    if _use_hip(w.norm):
        from . import hip
        return hip.general_delta(p, w, state, slot_ids, positions, meta,
                                 frag)
    return ref.general_delta(p, w, state, meta)


def ln_residual(x, y, norm: Optional[LayerNorm], mult, eps, scale=None,
                embed=None, tokens=None, rows=None, need_x=True, frag=False,
                then: Optional[LayerNorm] = None):
    """One pass between two matrix products, the norm after the sum:
    x' = norm(mult * x + scale * y), h = then(x'), or x' itself.  x is fp32
    [T, W], or None for the embedding rows of `tokens`; y a tensor, Partials
    or Branches of them, or None, and then x' = x; scale fp32 [W] or None;
    `rows` selects the rows to compute; frag returns h as FragRows.
    Returns (x', h)."""
    if _use_hip(embed):
        from . import hip
        return hip.ln_residual(x, y, norm, mult, eps, scale, embed, tokens,
                               rows, need_x, frag, then)
    return ref.ln_residual(x, y, norm, mult, eps, scale, embed, tokens, rows,
                           then)


def rms_residual(x, y, post, pre, mult, eps, embed=None, tokens=None,
                 embed_scale=1.0, rows=None, need_x=True, frag=False,
                 shift=None, tail=False, bare=False):
    """One pass between two matrix products:
    x' = x + mult * N(y) * post + shift, without `post` x + mult * y + shift;
    h = N(x') * pre, or x' itself without `pre`; N divides a row by its root
    mean square.  x is fp32 [T, W], or None for the scaled embedding rows of
    `tokens` (for nothing if `bare`); y a tensor, Partials, Weighted or None;
    shift fp32 [W] or None; `rows` selects the rows to compute; `tail`
    appends the token's embedding row to h; frag returns h as FragRows.
    Returns (x', h)."""
    if _use_hip(embed):
        from . import hip
        return hip.rms_residual(x, y, post, pre, mult, eps, embed, tokens,
                                embed_scale, rows, need_x, frag, shift=shift,
                                tail=tail, bare=bare)
    return ref.rms_residual(x, y, post, pre, mult, eps, embed, tokens,
                            embed_scale, rows, shift, tail, bare)


def rms_residual_route(x, y, post, mult, eps, moe, embed=None, tokens=None,
                       embed_scale=1.0, frag=False):
    """rms_residual without `pre`, and moe_route of the new operand:
    (x', h, (chosen, share))."""
    if _use_hip(embed):
        from . import hip
        return hip.rms_residual_route(x, y, post, mult, eps, moe, embed,
                                      tokens, embed_scale, frag)
    x, h = ref.rms_residual(x, y, post, None, mult, eps, embed, tokens,
                            embed_scale, None)
    return x, h, ref.moe_route(h, moe)


def qk_norm_append(p, cache, run, w: SigmoidAttn, q_norm, k_norm, eps,
                   slot_ids, positions):
    """Split the fused projection p (columns q | k | v; a tensor or
    Partials), RMS norm of all queries and of all keys of a token, append of
    keys and values to the run's paged pools.  -> queries [T, H, D'], rows
    filled up with zeros as the pool's are."""
    t = p.parts if isinstance(p, Partials) else p
    if _use_hip(t):
        from . import hip
        return hip.qk_norm_append(p, cache, run, w, q_norm, k_norm, eps,
                                  slot_ids, positions)
    return ref.qk_norm_append(p, cache, run, w, q_norm, k_norm, eps,
                              slot_ids, positions)


def sigmoid_attention(q, cache, run, w: SigmoidAttn, slot_ids, positions,
                      meta: AttnMeta, frag=False):
    """Causal attention with independent key weights over the run's paged
    keys and values; q as qk_norm_append returns it.  -> [T, H*V]."""
    if _use_hip(q):
        from . import hip
        return hip.sigmoid_attention(q, cache, run, w, slot_ids, positions,
                                     meta, frag)
    return ref.sigmoid_attention(q, cache, run, w, meta)


def moe_route(h, w: MoeWeights):
    """(experts int32 [T, top], strongest first; their shares fp32 of a
    softmax over all experts), router logits in fp32."""
    if _use_hip(w.router):
        from . import hip
        return hip.moe_route(h, w)
    return ref.moe_route(h, w)


def moe_experts(h, w: MoeWeights, chosen, share, packs=None) -> Weighted:
    """The chosen experts' outputs for every token, not yet added up.
    packs: packed copies of gate_up and down for decode."""
    if _use_hip(w.router):
        from . import hip
        return hip.moe_experts(h, w, chosen, share, packs or {})
    return ref.moe_experts(h, w, chosen, share)


def swiglu(gate_up, act="silu"):
    """act(gate) * up with act "silu" or "gelu_tanh"."""
    if _use_hip(gate_up):
        from . import hip
        return hip.swiglu(gate_up, act)
    return ref.swiglu(gate_up, act)


def gateup_swiglu(x, weight, packed_gu=None, act="silu"):
    """act = swiglu(x @ Wgu^T), or with another activation of the gate.
    On the decode path (M<=32) with a GU-packed copy this is ONE fused
    weight-streaming kernel; otherwise
    the library GEMM + the swiglu kernel.  (An MT2 variant for 33..64
    exists but measured BELOW the library at 64 users — its direct
    fragment x-loads double the scattered line traffic.)  FragRows go
    through the fused kernel at any batch and stay FragRows."""
    if isinstance(x, FragRows):
        from . import hip
        return hip.linear_gu_frag(x, packed_gu, weight.shape[0], act)
    if packed_gu is not None and x.shape[0] <= 32 and _use_hip(x):
        from . import hip
        if hip.USE_WSTREAM and x.dtype == torch.bfloat16 \
                and x.stride(1) == 1:
            return hip.linear_gu(x, packed_gu, weight.shape[0], glu=act)
    return swiglu(linear(x, weight), act)


def pack_weight_gu(w):
    """GU-interleaved packed copy for the fused gate_up+SwiGLU kernel."""
    if w.is_cuda:
        from . import hip
        if hip.available():
            return hip.pack_weight_gu(w)
    return None


# ---- fused-rmsnorm decode chain (GPU-only; the model gates on
# fused_chain availability — tp=1, decode, batch<=32) -----------------

def row_sumsq(x, out=None):
    """sq[m] = sum(x[m]**2) in fp32 (seeds the chain after embedding)."""
    if _use_hip(x):
        from . import hip
        return hip.row_sumsq(x, out)
    s = (x.float() ** 2).sum(-1)
    if out is not None:
        out.copy_(s)
        return out
    return s


def linear_fused(x, packed, N, bias=None, rstd=None, rstd_nt=0,
                 inv_h=0.0, eps=0.0, res=None, sq_out=None, y=None,
                 yfrag=0, K=None, xlds=None, M_frag=32):
    """Weight-streaming GEMM with the fused-chain epilogue/prologue:
    optional rmsnorm scaling of the raw-residual input (norm weight
    folded into the pack), in-place residual add (pass y=res) and
    sum-of-squares partial emission for the next GEMM's rstd.
    K given => x is a 32-row frag-layout buffer streamed linearly;
    yfrag => the output is emitted in frag layout."""
    from . import hip
    return hip.linear_packed(x, packed, bias, N, rstd=rstd,
                             rstd_nt=rstd_nt, inv_h=inv_h, eps=eps,
                             res=res, sq_out=sq_out, y=y, yfrag=yfrag,
                             K=K, xlds=xlds, M_frag=M_frag)


def fragify_sumsq(x, xf=None, sq=None):
    """Standard [M, H] -> 32-row frag layout + per-row sum of squares."""
    from . import hip
    return hip.fragify_sumsq(x, xf, sq)


def attention_decode_frag(q, cache, layer, meta):
    """Decode attention emitting its output in frag layout."""
    from . import hip
    return hip.attention_decode(q, cache, layer, meta, fragout=True)


def gu_fused(x, packed, N, rstd, rstd_nt, inv_h, eps, K=None, yfrag=0,
             M_frag=32):
    """rmsnorm -> gate_up GEMM -> SwiGLU, one kernel."""
    from . import hip
    return hip.linear_gu(x, packed, N, rstd=rstd, rstd_nt=rstd_nt,
                         inv_h=inv_h, eps=eps, K=K, yfrag=yfrag,
                         M_frag=M_frag)


def pack_weight_qkv_rope(w, nl, nkl):
    """Pair-ordered qkv pack for the fused RoPE/KV-append epilogue."""
    if w.is_cuda and w.shape[1] % 64 == 0:
        from . import hip
        if hip.available():
            return hip.pack_weight_qkv_rope(w, nl, nkl)
    return None


def qkv_rope_bias_order(bias, nl, nkl):
    """Reorder a qkv bias to match the pair-ordered pack."""
    from . import hip
    order = torch.tensor(hip.qkv_rope_order(nl, nkl), device=bias.device)
    return bias.index_select(0, order).contiguous()


def qkv_rope_fused(x, packed, N, bias_rp, cache, layer, positions, slots,
                   cos, sin, nl, nkl, rstd, rstd_nt, inv_h, eps,
                   K=None, M_real=32):
    """rmsnorm -> qkv GEMM -> RoPE -> paged KV append, one kernel."""
    from . import hip
    return hip.linear_qkv_rope(x, packed, N, bias_rp, cache, layer,
                               positions, slots, cos, sin, nl, nkl,
                               rstd, rstd_nt, inv_h, eps, K=K,
                               M_real=M_real)


def sample(logits, temperature, top_k, top_p, generator=None):
    # Sampler: torch ops compose on-GPU; custom fused kernel in ops/hip.py
    # handles the greedy + temperature paths.
    if _use_hip(logits):
        from . import hip
        return hip.sample(logits, temperature, top_k, top_p, generator)
    return ref.sample(logits, temperature, top_k, top_p, generator)
