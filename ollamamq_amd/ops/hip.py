"""ctypes bindings for the gfx950 HIP kernels (csrc/kernels/kernels.hip).

The extension is built IN-TREE (csrc/kernels/_kernels_gfx950.so) so the
.so travels with the repo snapshot to GPU boxes.  On a GPU box a missing
extension is a hard error — ops never fall back silently to eager PyTorch
(the GPU tests must exercise the native path).
"""
from __future__ import annotations

import ctypes
import os
from typing import NamedTuple, Optional

import torch

from . import reference as ref
from .interface import (LIGHTNING_CHUNK, AttnMeta, Branches, FragRows,
                        Partials, Weighted)

_LIB_PATH = os.path.join(
    os.path.dirname(os.path.dirname(os.path.abspath(__file__))),
    "csrc", "kernels", "_kernels_gfx950.so",
)

_lib = None
_load_err: Optional[str] = None


def _try_load():
    global _lib, _load_err
    if _lib is not None or _load_err is not None:
        return
    try:
        lib = ctypes.CDLL(_LIB_PATH, mode=ctypes.RTLD_GLOBAL)
    except OSError as e:
        _load_err = f"cannot load {_LIB_PATH}: {e}"
        return
    vp, i, f = ctypes.c_void_p, ctypes.c_int, ctypes.c_float
    lib.rmsnorm_residual_bf16.argtypes = [vp, vp, vp, vp, vp, i, i, f, vp]
    i64 = ctypes.c_int64
    lib.rope_bf16.argtypes = [vp, vp, vp, vp, vp, i, i, i, i, i64, i64, vp]
    lib.kv_append_bf16.argtypes = [vp, vp, vp, vp, vp, vp, vp,
                                   i, i, i, i, i, i64, vp]
    lib.paged_attn_bf16.argtypes = [vp, vp, vp, vp, vp, vp, vp, vp, vp,
                                    i, i, i, i, i, i, f, i64, vp]
    lib.swiglu_bf16.argtypes = [vp, vp, i, i, i, vp]
    lib.swiglu_f32.argtypes = lib.swiglu_bf16.argtypes
    lib.argmax_bf16.argtypes = [vp, vp, i, i, vp, vp, i, vp]
    lib.argmax_f32.argtypes = lib.argmax_bf16.argtypes
    lib.decode_attn_bf16.argtypes = [vp, vp, vp, vp, vp, vp, vp, vp, vp,
                                     i, i, i, i, i, f, i64, i, i, i, vp,
                                     i, vp]
    lib.skinny_gemm_bf16.argtypes = [vp, vp, vp, vp, i, i, i, i64, i, vp]
    lib.skinny_direct_bf16.argtypes = [vp, vp, vp, vp, i, i, i, i64, i, vp]
    lib.rope_append_bf16.argtypes = [vp, vp, vp, vp, vp, vp, vp, vp, vp, vp,
                                     i, i, i, i, i, i, i64, i64, i64, vp]
    lib.prefill_attn_bf16.argtypes = [vp, vp, vp, vp, vp, vp, vp, vp, vp,
                                      i, i, i, i, i, f, i64, i, vp]
    lib.embed_gather_bf16.argtypes = [vp, vp, vp, i, i, vp]
    lib.wstream_gemm_bf16.argtypes = [vp, vp, vp, vp, vp, i, i, i, i64, i,
                                      i, i, vp, i, f, f, vp, vp, i, vp]
    lib.wstream_pure_bf16.argtypes = [vp, vp, i, i, i, vp]
    lib.wstream_gu_bf16.argtypes = [vp, vp, vp, i, i, i, i64, i,
                                    vp, i, f, f, i, i, vp]
    lib.row_sumsq_bf16.argtypes = [vp, vp, i, i, vp]
    lib.fragify_sumsq_bf16.argtypes = [vp, vp, vp, i, i, vp]
    lib.sample_gumbel_bf16.argtypes = [vp, vp, vp, vp, vp, vp, i, i,
                                       vp, vp, i, vp]
    lib.decode_pure_bf16.argtypes = [vp, vp, vp, vp, vp, vp, i, i, i, i,
                                     i, i, vp]
    lib.wstream_qkv_rope_bf16.argtypes = [vp, vp, vp, vp, i, i, i, i64,
                                          vp, i, f, f, vp, vp, vp, vp,
                                          vp, vp, vp, i, i, i, i, i, vp]
    lib.dyt_residual.argtypes = [i, vp, vp, vp, vp, vp, vp, vp, i,
                                 vp, vp, f, vp, vp, f, vp, vp, vp, vp, vp,
                                 vp, vp, i, i, i, i, vp]
    lib.polynorm.argtypes = [i, vp, vp, vp, i, f, f, f, f, i, i, f, i, vp]
    lib.latent_append.argtypes = [i, vp, vp, i64, vp, vp, vp, vp,
                                  i, i, i, i, f, vp]
    lib.latent_gather.argtypes = [i, vp, vp, vp, vp, i, i, i, i, vp]
    rows = [vp, i, i, i64, i64]      # pointer, fp32?, parts, strides
    lib.head_gemm.argtypes = [i, vp, vp, vp, *rows, i, i, i, i, i, i64, i, i,
                              i, i, vp]
    lib.latent_mt.argtypes = [i, i, i, i]
    lib.latent_attn.argtypes = [i, vp, vp, vp, vp, vp, vp, vp, vp, vp,
                                i, i, i, i, i, i, i, f, i, i64, i64, i64, i,
                                vp]
    lib.latent_rope_append.argtypes = [i, vp, vp, *rows, vp, vp, vp, vp, vp,
                                       i, i, i, i, i, i, i, i, f, vp]
    lib.rope_qkv_append.argtypes = [i, vp, vp, vp, *rows, vp, vp, i, vp, vp,
                                    vp, i, i, i, i, i, i, i, i, i, vp]
    lib.softmax_rows.argtypes = [i, i, i]
    lib.softmax_step.argtypes = [i]
    lib.softmax_attn.argtypes = [i, i, vp, vp, vp, vp, vp, vp, vp, vp, vp,
                                 vp, i, i, i, i, i, i, i, i, i, i, i, i, i,
                                 f, vp, i, i, *rows, i, vp]
    lib.qkv_norm_rope.argtypes = [i, vp, vp, vp, *rows, vp, vp, vp, i, f, vp,
                                  i, vp, vp, vp, i, i, i, i, i, i, i, i, i,
                                  vp]
    lib.head_gate.argtypes = [i, vp, vp, f, vp, i, *rows, i, i, i, i, i, f, i,
                              vp]
    lib.ln_residual.argtypes = [i, vp, vp, vp, vp, vp, vp, i, i, i64, vp, i,
                                i, i64, vp, vp, f, vp, vp, vp, f, vp, vp, f,
                                vp, i, i, i, vp]
    lib.gated_rows.argtypes = [i, *rows, i, i, i, i, i, i, vp, i, vp, vp, vp,
                               vp, i, vp, vp, vp, vp, vp, vp, vp, vp, vp, i,
                               i, i, i, i, vp]
    lib.general_rows.argtypes = [i, *rows, i, i, i, vp, vp, vp, vp, vp, i, i,
                                 i, i, vp]
    delta = [vp, i64, i, i, i, i, vp, vp, i, vp, vp, vp, vp, vp, vp]
    lib.delta_step.argtypes = [i, i, vp, *delta, vp, i, i, i, i, i, vp, i,
                               vp, i64, i, f, i, vp]
    lib.delta_whole.argtypes = [i, i, i, i, i, i64]
    lib.delta_chunks.argtypes = [i, i, vp, vp, *delta, vp, i, vp, i, i, i, i,
                                 i, vp]
    lib.delta_scratch_floats.argtypes = [i, i, i, i]
    lib.delta_scratch_floats.restype = i64
    lib.rms_gate.argtypes = [i, vp, vp, vp, *rows, i, i, i, f, i, vp]
    lib.lightning_step.argtypes = [i, vp, *rows, i, i, i, i, vp, vp, vp, vp,
                                   vp, i, i, i, i, vp]
    lib.lightning_chunks.argtypes = [i, vp, vp, *rows, i, i, i, i, vp, vp, vp,
                                     vp, vp, vp, i, i, i, i, i, i, vp]
    lib.lightning_scratch.argtypes = [i, i, i, i]
    lib.lightning_scratch.restype = i64
    lib.flash_rows.argtypes = [i]
    lib.flash_attn.argtypes = [i, vp, vp, vp, vp, vp, vp, i64, i, vp, i, i,
                               i, i, i, i64, i64, i64, f, i, vp]
    lib.gla_step.argtypes = [i, vp, vp, i64, i, i, i, i, i, i, vp, vp, vp,
                             vp, vp, vp, vp, i, i, i, i, f, f, f, i, vp]
    lib.gla_chunks.argtypes = [i, vp, vp, vp, vp, i64, i, i, i, i, i, i,
                               vp, vp, vp, vp, vp, vp, vp, i, vp, i, i, i,
                               i, i, i, f, f, f, vp]
    lib.gla_scratch_floats.argtypes = [i, i, i]
    lib.gla_scratch_floats.restype = i64
    lib.rms_residual.argtypes = [i, vp, vp, vp, vp, vp, f, vp, i, i, i64,
                                 i64, vp, vp, vp, vp, f, f, vp, i, i, i, i,
                                 i, vp, vp, vp, i, i, vp]
    lib.qk_norm_append.argtypes = [i, vp, vp, vp, vp, i, i, i64, i64, vp, vp,
                                   vp, vp, vp, i, i, i, i, i, i, i, i, i, f,
                                   vp]
    lib.sigmoid_rows.argtypes = [i, i, i]
    lib.sigmoid_step.argtypes = [i]
    lib.sigmoid_attn.argtypes = [i, i, vp, vp, vp, vp, vp, vp, vp, vp, vp,
                                 i, i, i, i, i, i, i, i, i, i, i, i, i,
                                 f, f, vp, vp, vp, i, vp]
    lib.moe_route.argtypes = [i, vp, vp, vp, vp, i, i, i, i, i, vp]
    lib.moe_plan.argtypes = [vp, vp, vp, i, i, i, i, vp]
    lib.moe_mm.argtypes = [i, i, vp, vp, vp, vp, vp, i, i, i, i, vp]
    lib.moe_gemm.argtypes = [i, vp, vp, vp, vp, vp, i, i, i, i, vp]
    lib.moe_gemm_packed.argtypes = lib.moe_gemm.argtypes
    lib.moe_stream.argtypes = [i, vp, vp, vp, vp, vp, i, i, i, i, i, vp]
    for fn in ("rmsnorm_residual_bf16", "rope_bf16", "kv_append_bf16",
               "paged_attn_bf16", "swiglu_bf16", "argmax_bf16",
               "decode_attn_bf16", "skinny_gemm_bf16",
               "skinny_direct_bf16", "prefill_attn_bf16",
               "rope_append_bf16", "embed_gather_bf16",
               "wstream_gemm_bf16"):
        getattr(lib, fn).restype = ctypes.c_int
    _lib = lib


def _check(err: int, op: str):
    if err != 0:
        raise RuntimeError(f"HIP kernel launch failed in {op}: hipError {err}")


def available() -> bool:
    _try_load()
    return _lib is not None


def require():
    _try_load()
    if _lib is None:
        raise RuntimeError(
            "ollamamq_amd HIP extension missing on a GPU box: "
            f"{_load_err}. Build it with `python -m ollamamq_amd.build` "
            "(hipcc --offload-arch=gfx950)."
        )


def _stream():
    return ctypes.c_void_p(torch.cuda.current_stream().cuda_stream)


def _p(t: Optional[torch.Tensor]):
    return ctypes.c_void_p(0 if t is None else t.data_ptr())


# ---------------------------------------------------------------------------

def embedding(tokens, table):
    """out[t] = table[tokens[t]]: one gather kernel, int32 ids, no casts."""
    T = tokens.shape[0]
    V, H = table.shape
    if H % 8 or table.dtype != torch.bfloat16:
        return table.index_select(0, tokens.long())
    tok32 = tokens if tokens.dtype == torch.int32 else tokens.int()
    out = torch.empty((T, H), dtype=table.dtype, device=table.device)
    _check(_lib.embed_gather_bf16(_p(out), _p(table), _p(tok32), T, H,
                                  _stream()), "embed_gather")
    return out


def rmsnorm_residual(x, residual, weight, eps):
    T, H = x.shape
    y = torch.empty_like(x)
    res_out = torch.empty_like(x)
    _check(_lib.rmsnorm_residual_bf16(_p(y), _p(res_out), _p(x),
                                      _p(residual), _p(weight), T, H,
                                      float(eps), _stream()), "rmsnorm")
    return y, res_out


def _row_stride(t, D):
    # tolerate fused-QKV views: [T, H, D] with stride (S, D, 1)
    assert t.stride(2) == 1 and t.stride(1) == D, "head dim must be packed"
    return t.stride(0)


def rope(q, k, positions, cos, sin):
    T, Hq, D = q.shape
    Hk = k.shape[1]
    assert D == 128, "rope kernel specialized for head_dim=128"
    pos32 = positions if positions.dtype == torch.int32 else positions.int()
    _check(_lib.rope_bf16(_p(q), _p(k), _p(pos32), _p(cos), _p(sin),
                          T, Hq, Hk, D, _row_stride(q, D), _row_stride(k, D),
                          _stream()), "rope")


def kv_append(cache, layer, k, v, slot_ids, positions):
    T, KVH, D = k.shape
    kp, vp = _layer_ptrs(cache, layer)
    pos32 = positions if positions.dtype == torch.int32 else positions.int()
    slot32 = slot_ids if slot_ids.dtype == torch.int32 else slot_ids.int()
    assert _row_stride(k, D) == _row_stride(v, D)
    _check(_lib.kv_append_bf16(kp, vp, _p(k), _p(v), _p(slot32), _p(pos32),
                               _p(cache.page_table), T, KVH, D,
                               cache.page_size, cache.page_table.shape[1],
                               _row_stride(k, D), _stream()), "kv_append")


def rope_append(cache, layer, q, k, v, positions, slot_ids, cos, sin):
    """Fused RoPE (q,k in place) + paged append of rotated k and v."""
    T, Hq, D = q.shape
    KVH = k.shape[1]
    assert D == 128
    kp, vp = _layer_ptrs(cache, layer)
    pos32 = positions if positions.dtype == torch.int32 else positions.int()
    slot32 = slot_ids if slot_ids.dtype == torch.int32 else slot_ids.int()
    _check(_lib.rope_append_bf16(
        _p(q), _p(k), _p(v), kp, vp, _p(pos32), _p(slot32),
        _p(cache.page_table), _p(cos), _p(sin), T, Hq, KVH, D,
        cache.page_size, cache.page_table.shape[1],
        _row_stride(q, D), _row_stride(k, D), _row_stride(v, D),
        _stream()), "rope_append")


def _layer_ptrs(cache, layer):
    stride = cache.k_pool.stride(0) * cache.k_pool.element_size()
    return (ctypes.c_void_p(cache.k_pool.data_ptr() + layer * stride),
            ctypes.c_void_p(cache.v_pool.data_ptr() + layer * stride))


PREFILL_QT = 32


def _attn_plan(cache, meta, qt):
    """Device tile arrays for the attention launch, cached on the meta
    object (one build per forward, shared by every layer)."""
    key = f"_plan_{qt}"
    plan = getattr(meta, key, None)
    if plan is not None:
        return plan
    dev = meta.slot_ids.device
    if qt == 1:
        n = meta.slot_ids.shape[0]
        tile_slot = meta.slot_ids.int()
        tile_q0 = torch.arange(n, dtype=torch.int32, device=dev)
        tile_pos0 = (meta.seq_lens - 1).int()
        tile_rows = torch.ones(n, dtype=torch.int32, device=dev)
    else:
        slots = meta.slot_ids.tolist()
        lens = meta.seq_lens.tolist()
        cu = meta.cu_q.tolist()
        ts, tq, tp, tr = [], [], [], []
        for i, slot in enumerate(slots):
            qlen = cu[i + 1] - cu[i]
            start_pos = lens[i] - qlen
            for t0 in range(0, qlen, qt):
                rows = min(qt, qlen - t0)
                ts.append(slot)
                tq.append(cu[i] + t0)
                tp.append(start_pos + t0)
                tr.append(rows)
        tile_slot = torch.tensor(ts, dtype=torch.int32, device=dev)
        tile_q0 = torch.tensor(tq, dtype=torch.int32, device=dev)
        tile_pos0 = torch.tensor(tp, dtype=torch.int32, device=dev)
        tile_rows = torch.tensor(tr, dtype=torch.int32, device=dev)
    plan = (tile_slot, tile_q0, tile_pos0, tile_rows)
    setattr(meta, key, plan)
    return plan


def _attention(q, cache, layer, meta, qt):
    T, Hq, D = q.shape
    assert D == 128
    out = torch.empty_like(q)
    kp, vp = _layer_ptrs(cache, layer)
    tile_slot, tile_q0, tile_pos0, tile_rows = _attn_plan(cache, meta, qt)
    n_tiles = tile_slot.shape[0]
    if n_tiles == 0:
        return out
    _check(_lib.paged_attn_bf16(
        _p(out), _p(q), kp, vp, _p(cache.page_table),
        _p(tile_slot), _p(tile_q0), _p(tile_pos0), _p(tile_rows),
        n_tiles, qt, Hq, cache.n_kv_heads, cache.page_size,
        cache.page_table.shape[1], 1.0 / (D ** 0.5), _row_stride(q, D),
        _stream()), "paged_attn")
    return out


_scratch = {}


def _decode_scratch(S, Hq, split, dev):
    key = (S, Hq, split, str(dev))
    t = _scratch.get(key)
    if t is None:
        t = (torch.empty(S * Hq * split * 128, dtype=torch.float32,
                         device=dev),
             torch.empty(S * Hq * split * 2, dtype=torch.float32,
                         device=dev))
        _scratch[key] = t
    return t


def _combine_sem(S, KVH, dev):
    """Ticket counters for the in-launch split-K combine: zero-initialized
    once; the last-arriving block resets its counter, so the buffer is
    always all-zero between launches (guide G16 counter recipe)."""
    key = ("sem", S, KVH, str(dev))
    t = _scratch.get(key)
    if t is None:
        t = torch.zeros(S * KVH, dtype=torch.int32, device=dev)
        _scratch[key] = t
    return t


# staged KV chunk length (tokens) per pipeline stage; 32/64 compiled
# (the kernel scores one key per wave64 lane, so 64 is the ceiling).
# 64 wins for GQA groups >= 2 (sweep in NOTES.md); G=1 (MHA, Llama-2)
# takes 32 so the register-prefetch pipeline fits (NPF=8) — measured
# 142.9 -> 101.4 us at ctx 512 (see NOTES.md)
_CHUNK_ENV = os.environ.get("OLLAMAMQ_DECODE_CHUNK")


def _decode_chunk(G):
    if _CHUNK_ENV:
        return min(64, int(_CHUNK_ENV))
    return 32 if G == 1 else 64


def attention_decode(q, cache, layer, meta, fragout=False):
    """Flash-decoding: KV-split partials + exact online-softmax combine.

    The split factor targets ≥1024 workgroups so the memory-bound KV sweep
    fills the 256-CU chip (a bare (seq, kv-head) grid at batch 32 is 1
    workgroup/CU and runs at ~10% of HBM bandwidth).
    fragout: emit the output in the fused-chain 32-row frag layout (the
    o GEMM streams it linearly like packed weights)."""
    S, Hq, D = q.shape
    assert D == 128
    out = torch.empty((((S + 31) // 32) * 32 * Hq * D,)
                      if fragout else (S, Hq, D),
                      dtype=q.dtype, device=q.device)
    kp, vp = _layer_ptrs(cache, layer)
    kvh = cache.n_kv_heads
    # target ~1024 blocks; under graph capture max_kv is the pool's
    # max_ctx, so an unconditional max-split would freeze in dozens of
    # empty segments per sequence (measured: 5.55k -> 4.3k tok/s)
    want = max(1, 1024 // max(1, S * kvh))
    env = os.environ.get("OLLAMAMQ_DECODE_SPLIT")
    if env:                       # tuning override (tools/perf_decode.py)
        want = int(env)
    max_seg = max(1, (meta.max_kv + 63) // 64)
    split = int(min(want, max_seg, 32))
    o_part, ml_part = (None, None)
    op = mp = ctypes.c_void_p(0)
    sem = ctypes.c_void_p(0)
    if split > 1:
        o_part, ml_part = _decode_scratch(S, Hq, split, q.device)
        op, mp = _p(o_part), _p(ml_part)
        # in-launch combine measured WORSE (41.8 vs 29.3 us @ctx512 B32;
        # bench 5131 vs 5580): all S*split*KVH blocks pay the agent-scope
        # release fence (buffer_wbl2, ~1.7-6.5 us at 4 blocks/CU) to save
        # one 5 us combine launch. Kept for re-evaluation on shapes with
        # fewer, longer blocks.
        if os.environ.get("OLLAMAMQ_FUSED_COMBINE") == "1":
            sem = _p(_combine_sem(S, kvh, q.device))
    slot32 = meta.slot_ids.int() if meta.slot_ids.dtype != torch.int32 \
        else meta.slot_ids
    len32 = meta.seq_lens.int() if meta.seq_lens.dtype != torch.int32 \
        else meta.seq_lens
    _check(_lib.decode_attn_bf16(
        _p(out), op, mp, _p(q), kp, vp, _p(cache.page_table),
        _p(slot32), _p(len32), S, Hq, kvh, cache.page_size,
        cache.page_table.shape[1], 1.0 / (D ** 0.5), _row_stride(q, D),
        split, meta.window, _decode_chunk(Hq // kvh), sem,
        1 if fragout else 0, _stream()),
        "decode_attn")
    return out


def attention_mixed(q, cache, layer, meta):
    """Mixed batch: decode kernel over the first n_decode rows, MFMA
    prefill kernel over the remaining chunk rows — both write into one
    output tensor (sub-views share storage)."""
    T, Hq, D = q.shape
    nd = meta.n_decode
    out = torch.empty((T, Hq, D), dtype=q.dtype, device=q.device)
    # ---- decode part ----
    sub = getattr(meta, "_mixed_dec", None)
    if sub is None:
        sub = AttnMeta(
            mode="decode", slot_ids=meta.slot_ids[:nd],
            seq_lens=meta.seq_lens[:nd],
            cu_q=meta.cu_q[:nd + 1], logits_idx=None, max_q=1,
            max_kv=meta.max_kv, window=meta.window)
        meta._mixed_dec = sub
    if nd:
        out[:nd] = attention_decode(q[:nd], cache, layer, sub)
    # ---- prefill part (tiles over sequences nd..) ----
    plan = getattr(meta, "_mixed_plan", None)
    if plan is None:
        slots = meta.slot_ids[nd:].tolist()
        lens = meta.seq_lens[nd:].tolist()
        cu = meta.cu_q[nd:].tolist()
        dev = q.device
        ts, tq, tp, tr = [], [], [], []
        for i, slot in enumerate(slots):
            qlen = cu[i + 1] - cu[i]
            start_pos = lens[i] - qlen
            for t0 in range(0, qlen, PREFILL_QT):
                ts.append(slot)
                tq.append(cu[i] + t0)
                tp.append(start_pos + t0)
                tr.append(min(PREFILL_QT, qlen - t0))
        plan = (torch.tensor(ts, dtype=torch.int32, device=dev),
                torch.tensor(tq, dtype=torch.int32, device=dev),
                torch.tensor(tp, dtype=torch.int32, device=dev),
                torch.tensor(tr, dtype=torch.int32, device=dev))
        meta._mixed_plan = plan
    tile_slot, tile_q0, tile_pos0, tile_rows = plan
    n_tiles = tile_slot.shape[0]
    if n_tiles:
        kp, vp = _layer_ptrs(cache, layer)
        _check(_lib.prefill_attn_bf16(
            _p(out), _p(q), kp, vp, _p(cache.page_table),
            _p(tile_slot), _p(tile_q0), _p(tile_pos0), _p(tile_rows),
            n_tiles, Hq, cache.n_kv_heads, cache.page_size,
            cache.page_table.shape[1], 1.0 / (D ** 0.5),
            _row_stride(q, D), meta.window, _stream()), "prefill_attn")
    return out


def attention_prefill(q, cache, layer, meta):
    """MFMA flash prefill (prefill_attn.hip); set OLLAMAMQ_VALU_PREFILL=1
    to fall back to the VALU paged_attn path (A/B + debugging)."""
    if os.environ.get("OLLAMAMQ_VALU_PREFILL") == "1" \
            and not meta.window:   # VALU fallback predates sliding window
        return _attention(q, cache, layer, meta, 16)
    T, Hq, D = q.shape
    assert D == 128
    out = torch.empty((T, Hq, D), dtype=q.dtype, device=q.device)
    kp, vp = _layer_ptrs(cache, layer)
    tile_slot, tile_q0, tile_pos0, tile_rows = _attn_plan(cache, meta,
                                                          PREFILL_QT)
    n_tiles = tile_slot.shape[0]
    if n_tiles == 0:
        return out
    _check(_lib.prefill_attn_bf16(
        _p(out), _p(q), kp, vp, _p(cache.page_table),
        _p(tile_slot), _p(tile_q0), _p(tile_pos0), _p(tile_rows),
        n_tiles, Hq, cache.n_kv_heads, cache.page_size,
        cache.page_table.shape[1], 1.0 / (D ** 0.5), _row_stride(q, D),
        meta.window, _stream()), "prefill_attn")
    return out


# default 0 = library GEMMs everywhere: the fragment-direct kernel beats
# hipBLASLt on qkv/o in MICROBENCHES (L3-warm weights re-read 100x) but
# loses ~0.3 ms/step in the real serving loop where weights stream cold
# from HBM — honest A/B in bench.py decided this (5473 vs 5221 tok/s).
# The hand-written variants stay available via these env gates.
SKINNY_MAX_N = int(os.environ.get("OLLAMAMQ_SKINNY_MAX_N", "0"))
SKINNY_MAX_K = int(os.environ.get("OLLAMAMQ_SKINNY_MAX_K", "0"))

_gemm_scratch = {}


def _skinny_ksplit(N, K):
    """grid k-split: target >=768 blocks (~3/CU) so independent blocks
    hide each other's staging latency; kseg must stay a multiple of 256
    (even chunk count for the 2-deep pipeline)."""
    blocks = N // 32
    ks = 1
    while blocks * ks < 768 and ks < 8 and K % (256 * 2 * ks) == 0:
        ks *= 2
    return ks


def pack_weight(w):
    """Pre-pack a [N, K] bf16 weight into MFMA fragment order for the
    weight-streaming decode GEMM (wstream_gemm.hip): element W[n][k] with
    n = t*32+r, k = b*64 + j*16 + h*8 + e goes to 16-byte unit
    ((t*NB + b)*4 + j)*64 + (h*32 + r).  The kernel's loads then walk the
    buffer LINEARLY (full 128 B line per instruction, nt-tagged) — the fix
    for the 4x cold-line over-fetch of fragment-direct loads (NOTES r01).
    Returns None when the shape doesn't qualify."""
    N, K = w.shape
    if N % 32 or K % 64 or w.dtype != torch.bfloat16 \
            or not w.is_contiguous():
        return None
    p = w.reshape(N // 32, 32, K // 64, 4, 2, 8) \
         .permute(0, 2, 3, 4, 1, 5).contiguous()
    return p.view(-1)


def pack_weight_gu(w):
    """GU-interleaved pack of a fused [2F, K] gate_up weight: tile t holds
    gate rows f=t*16..t*16+16 then the matching 16 up rows, so the fused
    kernel's 32-column output tile pairs each gate with its up and the
    epilogue can apply SwiGLU in-register (wstream_gemm.hip GU=1)."""
    N, K = w.shape
    F = N // 2
    if N % 32 or F % 16 or K % 64 or w.dtype != torch.bfloat16 \
            or not w.is_contiguous():
        return None
    p = w.reshape(2, F // 16, 16, K // 64, 4, 2, 8) \
         .permute(1, 3, 4, 5, 0, 2, 6).contiguous()
    return p.view(-1)


GELU = {"silu": 0, "gelu_tanh": 1}      # activations of a gate


def linear_gu(x, packed, N, rstd=None, rstd_nt=0, inv_h=0.0, eps=0.0,
              K=None, yfrag=0, M_frag=32, glu="silu"):
    """act = swiglu(x @ Wgu^T) fused; N = 2F total weight rows; glu names
    the activation of the gate.
    With rstd: x is the raw residual and the epilogue applies the
    rmsnorm scale before SwiGLU (norm weight folded into the pack).
    K given => x is a frag-layout buffer (xlds=2); yfrag => the
    activation is emitted in frag layout for the down GEMM."""
    F = N // 2
    if K is None:
        M, K = x.shape
        xs = x.stride(0)
        xlds = (1 if N * K * 2 > (64 << 20) else 0) if M <= 32 else 0
    else:
        M, xs, xlds = M_frag, 0, 2
    act = torch.empty((M, F) if not yfrag
                      else (((M + 31) // 32) * 32 * F,),
                      dtype=x.dtype, device=x.device)
    _check(_lib.wstream_gu_bf16(
        _p(act), _p(x), _p(packed), M, N, K, xs, xlds,
        _p(rstd), rstd_nt, float(inv_h), float(eps), yfrag, GELU[glu],
        _stream()), "wstream_gu")
    return act


def _rope_pair_order(heads, d=128):
    """Output-row order pairing each head's RoPE halves: 16 lo dims then
    their 16 hi (d+64) dims, so every 32-row tile holds full rotation
    pairs for the fused qkv epilogue."""
    idx = []
    for h in range(heads):
        base = h * d
        for d0 in (0, 16, 32, 48):
            idx.extend(range(base + d0, base + d0 + 16))
            idx.extend(range(base + 64 + d0, base + 64 + d0 + 16))
    return idx


def qkv_rope_order(nl, nkl, d=128):
    """Row permutation for the whole fused qkv weight [q|k|v]."""
    q = _rope_pair_order(nl, d)
    k = [nl * d + i for i in _rope_pair_order(nkl, d)]
    v = [(nl + nkl) * d + i for i in range(nkl * d)]
    return q + k + v


def pack_weight_qkv_rope(w, nl, nkl):
    """Pair-ordered pack of the fused qkv weight for the RoPE epilogue."""
    order = torch.tensor(qkv_rope_order(nl, nkl), device=w.device)
    return pack_weight(w.index_select(0, order).contiguous())


def linear_qkv_rope(x, packed, N, bias_rp, cache, layer, positions,
                    slots, cos, sin, nl, nkl, rstd, rstd_nt, inv_h, eps,
                    K=None, M_real=32):
    """Fused rmsnorm -> qkv GEMM -> RoPE -> paged KV append: q returns
    rotated in the output's standard layout; k/v land in the pool."""
    if K is None:
        M, K = x.shape
        xs, xf = x.stride(0), 0
    else:
        M, xs, xf = M_real, 0, 1
    y = torch.empty((M, N), dtype=x.dtype, device=x.device)
    kp, vp = _layer_ptrs(cache, layer)
    pos32 = positions if positions.dtype == torch.int32 else positions.int()
    slot32 = slots if slots.dtype == torch.int32 else slots.int()
    _check(_lib.wstream_qkv_rope_bf16(
        _p(y), _p(x), _p(packed), _p(bias_rp), M, N, K, xs,
        _p(rstd), rstd_nt, float(inv_h), float(eps),
        _p(cos), _p(sin), _p(pos32), _p(slot32), _p(cache.page_table),
        kp, vp, nl, nkl, cache.page_size, cache.page_table.shape[1],
        xf, _stream()), "wstream_qkv_rope")
    return y


USE_WSTREAM = os.environ.get("OLLAMAMQ_NO_WSTREAM") != "1"


def _wstream_ksplit(N, K):
    """Measured rules (profiles/r02_gemm_sweep.md + in-graph A/B):
    * small weights (< 64 MB: qkv/o) are ramp/latency-floor-bound —
      fewer blocks with longer streams win (ks=1 beat every split);
    * big weights need >= 256 blocks to reach the full-chip stream rate
      (down at 128 blocks ran at half the chip: 41 vs 26 us);
    * uneven wave ranges (NB % 8ks != 0) cost ~10% tail imbalance
      (down ks3 measured worse than both ks2 and ks4);
    * very long (>16 iters) or very short (<4) per-wave streams lose."""
    tiles = N // 32
    nb = K // 64
    big = N * K * 2 > (64 << 20)
    best, best_cost = 1, 1 << 30
    for ks in range(1, 9):
        iters = nb // (ks * 8)
        if iters < 1:
            break
        cost = ks
        if nb % (ks * 8):
            cost += 16
        if big and tiles * ks < 256:
            cost += 24
        if iters < 4:
            cost += (4 - iters) * 8
        if iters > 16:
            cost += (iters - 16) * 2
        if cost < best_cost:
            best, best_cost = ks, cost
    return best


_WS_DEPTH = int(os.environ.get("OLLAMAMQ_WS_DEPTH", "1"))
_WS_XLDS = int(os.environ.get("OLLAMAMQ_WS_XLDS", "1"))
_WS_KS = os.environ.get("OLLAMAMQ_WS_KS")   # sweep override
# N above which the library GEMM wins (measured r02 sweep,
# profiles/r02_gemm_sweep.md: wstream beats hipBLASLt on the
# ramp-dominated small-N decode shapes qkv/o/down; on gate_up/logits the
# lib's big-grid kernels are closer to the stream ceiling than our
# x-load overhead allows — revisit after the x staging rework)
_WS_MAX_N = int(os.environ.get("OLLAMAMQ_WS_MAX_N", "16384"))


def linear_packed(x, packed, bias, N, ks=None, depth=None, xlds=None,
                  rstd=None, rstd_nt=0, inv_h=0.0, eps=0.0,
                  res=None, sq_out=None, y=None, yfrag=0, K=None,
                  M_frag=32):
    """y = x @ W^T via the weight-streaming kernel over pre-packed W.

    Fused-chain extras (decode, M<=32): `rstd`/`rstd_nt`/`inv_h`/`eps`
    apply rmsnorm scaling of the raw-residual input x (norm weight must
    be folded into the pack); `res` adds the residual stream into the
    output (pass y=res for the in-place residual update) and `sq_out`
    emits per-tile sum-of-squares partials for the next GEMM."""
    if K is None:
        M, K = x.shape
        xs = x.stride(0)
    else:                       # frag-layout x: flat buffer, xlds==2
        M = M_frag
        xs = 0
    if y is None:
        y = torch.empty((((M + 31) // 32) * 32 * N,) if yfrag
                        else (M, N), dtype=x.dtype, device=x.device)
    if ks is None:
        per_k = os.environ.get(f"OLLAMAMQ_WS_KS_{K}")   # per-shape tuning
        if per_k:
            ks = int(per_k)
        else:
            ks = int(_WS_KS) if _WS_KS else _wstream_ksplit(N, K)
    if rstd is not None:
        ks = 1            # rstd fusion requires ks == 1
    part = ctypes.c_void_p(0)
    if ks > 1:
        key = ("ws", M, N, ks, str(x.device))
        t = _gemm_scratch.get(key)
        if t is None:
            t = torch.empty(ks * M * N, dtype=torch.float32,
                            device=x.device)
            _gemm_scratch[key] = t
        part = _p(t)
    if xlds is None:
        # measured (profiles/r02_gemm_sweep.md): LDS x-staging pays on
        # long streams (down/gate_up/logits), the direct fragment load
        # wins on the short ramp-bound ones (qkv/o)
        xlds = (_WS_XLDS if M <= 32 and N * K * 2 > (64 << 20) else 0)
    _check(_lib.wstream_gemm_bf16(
        _p(y), part, _p(x), _p(packed), _p(bias), M, N, K, xs,
        ks, depth if depth is not None else _WS_DEPTH, xlds,
        _p(rstd), rstd_nt, float(inv_h), float(eps), _p(res), _p(sq_out),
        yfrag, _stream()), "wstream_gemm")
    return y


def fragify_sumsq(x, xf=None, sq=None):
    """Standard [M, H] -> 32-row frag layout + per-row sum of squares
    (seeds the fused decode chain after the embedding gather)."""
    M, H = x.shape
    if xf is None:
        xf = torch.empty(((M + 31) // 32) * 32 * H, dtype=x.dtype,
                         device=x.device)
    if sq is None:
        sq = torch.empty(M, dtype=torch.float32, device=x.device)
    _check(_lib.fragify_sumsq_bf16(_p(xf), _p(sq), _p(x), M, H,
                                   _stream()), "fragify_sumsq")
    return xf, sq


def row_sumsq(x, out=None):
    """sq[m] = sum(x[m]**2) fp32 — seeds the fused-rmsnorm chain."""
    M, H = x.shape
    if out is None:
        out = torch.empty(M, dtype=torch.float32, device=x.device)
    _check(_lib.row_sumsq_bf16(_p(out), _p(x), M, H, _stream()),
           "row_sumsq")
    return out


def wstream_pure(packed, N, K, ks):
    """Bandwidth diagnostic: the GEMM's weight stream alone."""
    sink = torch.zeros(1, dtype=torch.float32, device=packed.device)
    _check(_lib.wstream_pure_bf16(_p(sink), _p(packed), N, K, ks,
                                  _stream()), "wstream_pure")
    return sink


def linear(x, weight, bias=None, packed=None):
    if isinstance(x, FragRows):
        assert bias is None
        return _linear_frag(x, weight.shape[0], packed, False)
    M, K = x.shape
    N = weight.shape[0]
    if packed is not None and USE_WSTREAM and M <= 64 \
            and (N <= _WS_MAX_N or N >= 65536) \
            and x.dtype == torch.bfloat16 and x.stride(1) == 1:
        return linear_packed(x, packed, bias, N)
    # gated to the shapes where the hand-written kernel beats hipBLASLt
    # (measured tools/perf_gemm.py); widen via env as the kernel improves
    if bias is None and M <= 32 and K % 256 == 0 and N % 32 == 0 \
            and N <= SKINNY_MAX_N and K <= SKINNY_MAX_K \
            and x.dtype == torch.bfloat16 and weight.stride(1) == 1:
        y = torch.empty((M, N), dtype=x.dtype, device=x.device)
        assert x.stride(1) == 1
        direct = os.environ.get("OLLAMAMQ_SKINNY_STAGED") != "1"
        if direct:
            # per-wave k extent must be a multiple of 64
            ks = 1
            blocks = N // 32
            while blocks * ks < 768 and ks < 8 and K % (ks * 2 * 512) == 0:
                ks *= 2
            if K % (ks * 512) != 0:
                return torch.nn.functional.linear(x, weight)
        else:
            ks = _skinny_ksplit(N, K)
        part = ctypes.c_void_p(0)
        if ks > 1:
            key = (M, N, ks, str(x.device))
            t = _gemm_scratch.get(key)
            if t is None:
                t = torch.empty(ks * M * N, dtype=torch.float32,
                                device=x.device)
                _gemm_scratch[key] = t
            part = _p(t)
        fn = _lib.skinny_direct_bf16 if direct else _lib.skinny_gemm_bf16
        _check(fn(_p(y), part, _p(x), _p(weight),
                  M, N, K, x.stride(0), ks, _stream()), "skinny_gemm")
        return y
    return torch.nn.functional.linear(x, weight, bias)


def swiglu(gate_up, act="silu"):
    T, F2 = gate_up.shape
    F = F2 // 2
    out = torch.empty((T, F), dtype=gate_up.dtype, device=gate_up.device)
    f32 = _is_f32(gate_up)
    assert gate_up.is_contiguous() and (f32 or F % 8 == 0)
    fn = _lib.swiglu_f32 if f32 else _lib.swiglu_bf16
    _check(fn(_p(out), _p(gate_up), T, F, GELU[act], _stream()),
           "swiglu")
    return out


# ---------------------------------------------------------------------------
# dynamic-tanh blocks, latent attention, gated linear attention: every kernel
# exists for bf16 and for true fp32

def _is_f32(t):
    if t.dtype not in (torch.float32, torch.bfloat16):
        raise TypeError(f"kernels take float32 or bfloat16, not {t.dtype}")
    return int(t.dtype == torch.float32)


def _i32(t):
    return t if t.dtype == torch.int32 else t.int()


def _frag_rows(M, cols, like):
    """Buffer of an activation in fragment layout: 32-row halves."""
    return FragRows(torch.empty(-(-M // 32) * 32 * cols,
                                dtype=torch.bfloat16, device=like.device),
                    M, cols)


def _parts_ksplit(N, K, most=8):
    """Split for a product whose consumer folds the partial sums: the one
    that loads the 256 CUs most evenly, smaller if nearly as good."""
    tiles, nb = N // 32, K // 64
    best, best_eff = 1, 0.0
    for ks in range(1, most + 1):
        if nb < ks * 8:
            break
        n = tiles * ks
        eff = n / (256 * -(-n // 256))
        if eff > best_eff + 0.04:
            best, best_eff = ks, eff
    return best


def _linear_frag(x, N, packed, parts, most=8):
    """Weight-streaming product of an activation in fragment layout."""
    M, K = x.rows, x.cols
    ks = _parts_ksplit(N, K, most) if parts else _wstream_ksplit(N, K)
    y = part = None
    if ks > 1:
        part = torch.empty((ks, M, N), dtype=torch.float32,
                           device=packed.device)
    if ks == 1 or not parts:
        y = torch.empty((M, N), dtype=torch.bfloat16, device=packed.device)
    _check(_lib.wstream_gemm_bf16(
        _p(y), _p(part), _p(x.buf), _p(packed), _p(None), M, N, K, 0, ks,
        _WS_DEPTH, 2, _p(None), 0, 0.0, 0.0, _p(None), _p(None), 0,
        _stream()), "wstream_gemm")
    return y if y is not None else Partials(part)


def linear_f32(x, weight, packed=None):
    """A product whose consumer takes fp32: partial sums, also if there is
    only one, or the library's fp32 result."""
    N = weight.shape[0]
    if isinstance(x, FragRows):
        M, K = x.rows, x.cols
        part = torch.empty((_parts_ksplit(N, K), M, N), dtype=torch.float32,
                           device=weight.device)
        _check(_lib.wstream_gemm_bf16(
            _p(None), _p(part), _p(x.buf), _p(packed), _p(None), M, N, K, 0,
            part.shape[0], _WS_DEPTH, 2, _p(None), 0, 0.0, 0.0, _p(None),
            _p(None), 0, _stream()), "wstream_gemm")
        return Partials(part)
    if x.dtype == torch.float32:
        return torch.nn.functional.linear(x, weight)
    return torch.mm(x, weight.t(), out_dtype=torch.float32)


def linear_gu_frag(x, packed, N, glu="silu"):
    """linear_gu of an activation in fragment layout, and so its result."""
    act = linear_gu(x.buf, packed, N, K=x.cols, yfrag=1, M_frag=x.rows,
                    glu=glu)
    return FragRows(act, x.rows, N // 2)


def linear_parts(x, weight, packed=None, most=8):
    """Decode: the weight-streaming product, left as split-K partial sums
    where it splits (the next kernel folds them in)."""
    N = weight.shape[0]
    if isinstance(x, FragRows):
        return _linear_frag(x, N, packed, True, most)
    M, K = x.shape
    if packed is not None and USE_WSTREAM and M <= 64 and N <= _WS_MAX_N \
            and x.dtype == torch.bfloat16 and x.stride(1) == 1:
        ks = int(_WS_KS) if _WS_KS else _wstream_ksplit(N, K)
        if 1 < ks <= most:
            part = torch.empty((ks, M, N), dtype=torch.float32,
                               device=x.device)
            xlds = (_WS_XLDS if M <= 32 and N * K * 2 > (64 << 20) else 0)
            _check(_lib.wstream_gemm_bf16(
                _p(None), _p(part), _p(x), _p(packed), _p(None), M, N, K,
                x.stride(0), ks, _WS_DEPTH, xlds, _p(None), 0, 0.0, 0.0,
                _p(None), _p(None), 0, _stream()), "wstream_gemm")
            return Partials(part)
    return linear(x, weight, packed=packed)


def _row_seq(meta):
    """Sequence index of every row of a varlen batch (cached on the meta)."""
    t = getattr(meta, "_row_seq", None)
    if t is None:
        _, q_lens, _ = meta.layout()
        t = torch.repeat_interleave(
            torch.arange(len(q_lens), dtype=torch.int32),
            torch.tensor(q_lens)).to(meta.slot_ids.device)
        meta._row_seq = t
    return t


def dyt_residual(x, y, post, pre, shift, embed, tokens, rows, need_x,
                 frag=False):
    parts = y.parts if isinstance(y, Partials) else None
    yt = None if parts is not None else y
    W = pre.w.shape[0]
    if x is not None:
        T_in = x.shape[0]
        assert x.dtype == torch.float32 and x.is_contiguous()
    else:
        T_in = tokens.shape[0]
    dtype = embed.dtype
    assert yt is None or (yt.shape == (T_in, W) and yt.is_contiguous()
                          and yt.dtype == dtype)
    assert parts is None or parts.shape[1:] == (T_in, W)
    n = T_in if rows is None else rows.shape[0]
    if frag:
        assert dtype == torch.bfloat16 and W % 64 == 0
        res = _frag_rows(n, W, pre.w)
        h = res.buf
    else:
        res = h = torch.empty((n, W), dtype=dtype, device=pre.w.device)
    if x is not None and y is None and rows is None:
        x_out, write = x, None               # nothing to add
    else:
        x_out = write = (torch.empty((n, W), dtype=torch.float32,
                                     device=pre.w.device)
                         if need_x else None)
    mix = prev = slot = pos = row_seq = cu = None
    if shift is not None:
        assert rows is None
        mix, prev = shift.mix, shift.prev
        slot, pos = _i32(shift.slot_ids), _i32(shift.positions)
        if not shift.meta.one_each:
            row_seq, cu = _row_seq(shift.meta), shift.meta.cu_q
            assert cu.dtype == torch.int32
    tok = None if tokens is None else _i32(tokens)
    z = post if post is not None else pre
    if n == 0:
        return x_out, res
    _check(_lib.dyt_residual(
        _is_f32(h), _p(write), _p(h), _p(x), _p(embed), _p(tok), _p(yt),
        _p(parts), 0 if parts is None else parts.shape[0],
        _p(z.w), _p(z.b), z.alpha, _p(pre.w), _p(pre.b), pre.alpha,
        _p(mix), _p(prev), _p(slot), _p(pos), _p(row_seq), _p(cu), _p(rows),
        n, T_in, W, int(frag), _stream()), "dyt_residual")
    return x_out, res


def polynorm(z, coef, eps, frag=False):
    parts = z.parts if isinstance(z, Partials) else None
    T, F = (z if parts is None else parts[0]).shape
    dtype = torch.bfloat16 if parts is not None else z.dtype
    like = z if parts is None else parts
    if frag:
        assert dtype == torch.bfloat16 and F % 64 == 0
        res = _frag_rows(T, F, like)
        out = res.buf
    else:
        res = out = torch.empty((T, F), dtype=dtype, device=like.device)
    assert parts is not None or z.is_contiguous()
    _check(_lib.polynorm(
        _is_f32(out), _p(out), _p(None if parts is not None else z),
        _p(parts), 0 if parts is None else parts.shape[0], *coef, T, F,
        float(eps), int(frag), _stream()), "polynorm")
    return res


def latent_append(cache, run, d, weight, slot_ids, positions, eps):
    T, R = d.shape
    pool = cache.latent_pool[run]
    assert d.stride(1) == 1 and pool.dtype == d.dtype and pool.shape[2] == R
    _check(_lib.latent_append(
        _is_f32(d), _p(pool), _p(d), d.stride(0), _p(weight),
        _p(_i32(slot_ids)), _p(_i32(positions)), _p(cache.page_table), T, R,
        cache.page_size, cache.page_table.shape[1], float(eps), _stream()),
        "latent_append")


def _rows(p):
    """A projection, or the partial sums of one, as the kernels take it:
    (pointer, fp32?, parts, stride of a part, stride of a row)."""
    if p is None:
        return _p(None), 0, 1, 0, 0
    t = p.parts if isinstance(p, Partials) else p
    assert t.stride(-1) == 1
    f32 = int(t.dtype == torch.float32)
    if isinstance(p, Partials):
        return _p(t), f32, t.shape[0], t.stride(0), t.stride(1)
    return _p(t), f32, 1, 0, t.stride(0)


def _cols(p):
    return (p.parts if isinstance(p, Partials) else p).shape[-1]


def head_gemm(x, w, out, frag=False, tail=0, gate=None):
    """out[t, h] = w[h] @ x[t, h, :K]; x [T, H, >= K] (rows may be strided);
    frag: out is the buffer of a FragRows.  Wider rows of `out` end in `tail`
    values from behind the inputs, then zeros; gate: Columns whose sigmoid
    multiplies the result."""
    T, H, wide = x.shape
    N, K = w.shape[1:]
    os = N if frag else out.shape[2]
    assert w.shape[0] == H and w.is_contiguous() and wide >= K + tail \
        and (frag or out.shape == (T, H, os)) and out.is_contiguous() \
        and x.stride(2) == 1 and os >= N + tail
    gp, og = (None, 0) if gate is None else gate
    assert gp is None or og + H * N <= _cols(gp)
    if T:
        _check(_lib.head_gemm(_is_f32(x), _p(out), _p(x), _p(w), *_rows(gp),
                              og, T, H, N, K, x.stride(0),
                              x.stride(1) if H > 1 else wide, os, tail,
                              int(frag), _stream()), "head_gemm")
    return out


LATENT_MAX_R = 1024       # absorbed kernel: latent width
LATENT_SPLIT_MAX = 64     # and context segments
FLASH_MAX = 256           # expanded kernel: key and value widths
EXPAND_BYTES = 1 << 30    # expanded keys and values held at a time


def _absorbs(n, kv, H, D, E, V, R, KW, window):
    """Whether n queries after kv - n tokens attend in latent space: the
    expanded form pays R*(D+V) once per key it needs, the absorbed one KW+R
    instead of D+E+V for every (query, key).  D, E: unrotated and rotated key
    width."""
    if KW > LATENT_MAX_R:
        return False
    if max(D + E, V) > FLASH_MAX or n < 16:
        return True
    seen = min(kv, window) if window else kv
    keys = min(kv, n + window - 1) if window else kv
    return n * seen * (KW + R - D - E - V) < keys * R * (D + V)


def _latent_plan(meta, w, KW, f32, dev):
    """Batch layout for one attention shape, shared by the layers that have
    it: leading sequences attend in latent space, the rest expanded."""
    H, D, R = w.uk.shape
    V, E, window = w.uv.shape[1], w.rot_dim, w.window
    key = f"_latent_{H}_{D}_{E}_{V}_{R}_{window}"
    plan = getattr(meta, key, None)
    if plan is not None:
        return plan
    slots, q_lens, kv_lens = meta.layout()
    M = 16 * _lib.latent_mt(f32, H, R, KW)
    nd = meta.n_single
    i, row, items = nd, nd, []
    kv_absorbed = 0
    while i < len(slots) and _absorbs(q_lens[i], kv_lens[i], H, D, E, V, R,
                                      KW, window):
        lo, hi = row * H, (row + q_lens[i]) * H
        items += [(r, min(M, hi - r)) for r in range(lo, hi, M)]
        kv_absorbed = max(kv_absorbed, kv_lens[i])
        row += q_lens[i]
        i += 1
    n_absorbed = row
    QT = _lib.flash_rows(f32)
    esz = 4 if f32 else 2
    groups = []            # (gather rows, tiles, padded keys) per batch
    gather, tiles, kv0 = [], [], 0

    def flush():
        nonlocal gather, tiles, kv0
        if tiles:
            groups.append((
                torch.tensor(gather, dtype=torch.int32).to(dev),
                torch.tensor(tiles, dtype=torch.int32).to(dev), kv0))
        gather, tiles, kv0 = [], [], 0

    while i < len(slots):
        n, kv = q_lens[i], kv_lens[i]
        # whole groups of 64 positions from the first one a query sees
        lo = max(0, kv - n + 1 - window) // 64 * 64 if window else 0
        for b in range(lo, kv, 64):
            gather.append((slots[i], b, min(64, kv - b)))
        for t in range(0, n, QT):
            tiles.append((row + t, kv - n + t, min(QT, n - t), kv0 - lo))
        row += n
        kv0 += (kv - lo + 63) // 64 * 64
        i += 1
        if kv0 * H * (D + V) * esz > EXPAND_BYTES:
            flush()
    flush()
    dev_items = torch.tensor(items, dtype=torch.int32).to(dev) \
        if items else None
    plan = (n_absorbed, dev_items, kv_absorbed, groups)
    setattr(meta, key, plan)
    return plan


def _latent_absorbed(o, q, cache, run, slots, pos, H, w, items, n_items,
                     per_seq, row0, rows, max_kv):
    """One launch of the absorbed kernel over rows row0.. of q / o."""
    f32 = _is_f32(q)
    total, KW = q.shape
    R = o.shape[1]
    seen = min(max_kv, w.window + 63) if w.window else max_kv
    # one block a CU: more segments would only write more partial results
    split = int(max(1, min(256 // n_items, (seen + 63) // 64,
                           LATENT_SPLIT_MAX)))
    op = ml = None
    if split > 1:
        op = torch.empty((split, total, R), dtype=q.dtype, device=q.device)
        ml = torch.empty((split, total, 2), dtype=torch.float32,
                         device=q.device)
    pool = cache.latent_pool[run]
    assert pool.dtype == q.dtype and pool.shape[2] == KW
    _check(_lib.latent_attn(
        f32, _p(o), _p(op), _p(ml), _p(q), _p(pool), _p(cache.page_table),
        _p(slots), _p(pos), _p(items), n_items, per_seq, H, R, KW,
        cache.page_size, cache.page_table.shape[1], float(w.scale),
        w.window, total, row0, rows, split, _stream()), "latent_attn")


def latent_attention(q, cache, run, w, slot_ids, positions, meta,
                     frag=False, gate=None):
    H, D, R = w.uk.shape
    V, E = w.uv.shape[1], w.rot_dim
    T, DD = q.shape[0], D + E
    f32 = _is_f32(q)
    pool = cache.latent_pool[run]
    KW = pool.shape[2]
    assert q.shape[1] == H * DD and KW >= R + E
    if KW > LATENT_MAX_R and (max(DD, V) > FLASH_MAX or meta.n_single):
        raise ValueError(f"latent attention with rank {R}, head widths "
                         f"{DD}/{V}: no kernel")
    assert not frag or meta.one_each
    if frag:
        res = _frag_rows(T, H * V, q)
        out = res.buf
    else:
        out = torch.empty((T, H, V), dtype=q.dtype, device=q.device)
    slots, pos = _i32(slot_ids), _i32(positions)
    nd = meta.n_single
    if meta.one_each:
        n_abs, items, kv_abs, groups = T, None, 0, []
    else:
        n_abs, items, kv_abs, groups = _latent_plan(meta, w, KW, f32,
                                                    q.device)
    if n_abs:
        qa = q[:n_abs].unflatten(1, (H, DD))
        lat = torch.empty((n_abs, H, KW), dtype=q.dtype, device=q.device)
        head_gemm(qa, w.uk_t, lat, tail=E)
        lat = lat.view(n_abs * H, KW)
        o = torch.empty((n_abs * H, R), dtype=q.dtype, device=q.device)
        if nd:
            per = -(-H // (16 * _lib.latent_mt(f32, H, R, KW)))
            _latent_absorbed(o, lat, cache, run, slots, pos, H, w, None,
                             nd * per, per, 0, nd * H, meta.max_kv)
        if items is not None:
            _latent_absorbed(o, lat, cache, run, slots, pos, H, w, items,
                             items.shape[0], 1, nd * H, (n_abs - nd) * H,
                             kv_abs)
        head_gemm(o.view(n_abs, H, R), w.uv, out if frag else out[:n_abs],
                  frag, gate=gate)
        if frag:
            return res
    g, og = (None, 0) if gate is None else gate
    if groups and isinstance(g, Partials):
        g, og = g.parts[:, :, og:og + H * V].sum(0).to(q.dtype), 0
    assert g is None or not groups or (g.dtype == q.dtype
                                       and g.stride(1) == 1)
    for gather, tiles, kv in groups:
        c = torch.empty((kv, KW), dtype=q.dtype, device=q.device)
        _check(_lib.latent_gather(
            f32, _p(c), _p(pool), _p(cache.page_table), _p(gather),
            gather.shape[0], KW, cache.page_size, cache.page_table.shape[1],
            _stream()), "latent_gather")
        lat = c[:, :R]
        k = torch.nn.functional.linear(lat, w.uk.view(H * D, R))
        vt = torch.mm(w.uv.view(H * V, R), lat.t())
        _check(_lib.flash_attn(
            f32, _p(out), _p(q), _p(k), _p(c[:, R:] if E else None), _p(vt),
            _p(g), 0 if g is None else g.stride(0), og, _p(tiles),
            tiles.shape[0], H, D, E, V, q.stride(0), KW, kv, float(w.scale),
            w.window, _stream()), "flash_attn")
    return out.view(T, H * V)


def latent_rope_append(p, cache, run, w, norm, eps, rope, slot_ids,
                       positions):
    H, D, R = w.uk.shape
    E, pool, T = w.rot_dim, cache.latent_pool[run], slot_ids.shape[0]
    assert rope.dims == E and rope.table.shape == (rope.table.shape[0], E) \
        and rope.table.shape[0] >= cache.max_ctx and norm.numel() == R \
        and _cols(p) >= H * (D + E) + R + E
    q = torch.empty((T, H * (D + E)), dtype=pool.dtype, device=pool.device)
    rows = _rows(p)
    assert rows[1] or pool.dtype == torch.bfloat16
    if T:
        _check(_lib.latent_rope_append(
            _is_f32(q), _p(q), _p(pool), *rows, _p(norm), _p(rope.table),
            _p(_i32(slot_ids)), _p(_i32(positions)), _p(cache.page_table), T,
            H, D, E, R, pool.shape[2], cache.page_size,
            cache.page_table.shape[1], float(eps), _stream()),
            "latent_rope_append")
    return q


GLA_STEP_TOKENS = 4       # portions up to this walk token by token
GLA_CHUNK_MAX = (512, 256)   # key width and low rank the chunk kernels take


def _chunk_plan(meta, dev, step_tokens):
    """Layout of a recurrence: portions of up to `step_tokens` tokens at the
    front walk token by token, the rest in chunks of 64."""
    key = f"_chunk_plan_{step_tokens}"
    plan = getattr(meta, key, None)
    if plan is not None:
        return plan
    _, q_lens, _ = meta.layout()
    nd = meta.n_single
    i, row, spans = nd, nd, []
    while i < len(q_lens) and q_lens[i] <= step_tokens:
        spans.append((row, q_lens[i]))
        row += q_lens[i]
        i += 1
    base, chunks, seqs = row, [], []
    for n in q_lens[i:]:
        seqs.append((len(chunks), (n + 63) // 64))
        chunks += [(row + t, min(64, n - t)) for t in range(0, n, 64)]
        row += n
    t32 = lambda x: torch.tensor(x, dtype=torch.int32).to(dev) \
        if x else None
    plan = (t32(spans), t32(chunks), t32(seqs), base, row - base)
    setattr(meta, key, plan)
    return plan


def gla(p, w, state, slot_ids, positions, meta, frag=False):
    T = p.shape[0]
    H, D, V = w.heads, w.dim, w.vdim
    assert p.stride(1) == 1 and state.dtype == torch.float32 \
        and state.shape[1:] == (H, D, V) and w.a2.dtype == p.dtype
    assert max(w.offsets) + w.rank <= p.shape[1]
    assert not frag or meta.one_each
    if frag:
        res = _frag_rows(T, H * V, p)
        out = res.buf
    else:
        res = out = torch.empty((T, H * V), dtype=p.dtype, device=p.device)
    slots, pos = _i32(slot_ids), _i32(positions)
    f32 = _is_f32(p)
    head = (_p(p), p.stride(0), *w.offsets, w.rank, _p(w.a2), _p(w.a2_b),
            _p(w.norm), _p(state), _p(slots), _p(pos))
    tail = (H, D, V, D ** -0.5, 1.0 / w.tau, float(w.eps))
    nd = meta.n_single
    if nd:
        _check(_lib.gla_step(f32, _p(out), *head, _p(None), nd, *tail,
                             int(frag), _stream()), "gla_step")
    if meta.one_each:
        return res
    chunked = D <= GLA_CHUNK_MAX[0] and w.rank <= GLA_CHUNK_MAX[1]
    spans, chunks, seqs, base, rows = _chunk_plan(
        meta, p.device, GLA_STEP_TOKENS if chunked else 1 << 62)
    if spans is not None:
        _check(_lib.gla_step(f32, _p(out), *head, _p(spans),
                             spans.shape[0], *tail, 0, _stream()), "gla_step")
    if chunks is not None:
        nc = chunks.shape[0]
        scr = torch.empty(_lib.gla_scratch_floats(nc, H, D),
                          dtype=torch.float32, device=p.device)
        o = torch.empty(rows * H * V, dtype=torch.float32, device=p.device)
        _check(_lib.gla_chunks(
            f32, _p(out), _p(scr), _p(o), *head, _p(chunks), nc, _p(seqs),
            seqs.shape[0], base, rows, *tail, _stream()), "gla_chunks")
    return out


LIGHTNING_STEP_TOKENS = 4    # portions up to this walk token by token
LIGHTNING_MAX_D = 256        # key width the chunk kernels take


def lightning(p, w, state, slot_ids, positions, meta, frag=False):
    H, D, V = w.heads, w.dim, w.vdim
    rows = _rows(p)
    t = p.parts if isinstance(p, Partials) else p
    T, dtype = t.shape[-2], torch.bfloat16 if isinstance(p, Partials) \
        else p.dtype
    f32 = int(dtype == torch.float32)
    oq, ok, ov, og = w.offsets
    assert state.dtype == torch.float32 and state.is_contiguous() \
        and state.shape[1:] == (H, D, V) \
        and (w.norm is None or w.norm.numel() == H * V) \
        and w.powers.shape == (H, LIGHTNING_CHUNK + 1) \
        and w.powers.is_contiguous() \
        and max(oq + H * D, ok + H * D, ov + H * V, og + H * V) <= t.shape[-1]
    assert not frag or meta.one_each
    o = torch.empty((T, H * V), dtype=torch.float32, device=t.device)
    slots, pos = _i32(slot_ids), _i32(positions)
    head = (*rows, oq, ok, ov, int(w.act), _p(w.powers), _p(state),
            _p(slots), _p(pos))
    nd = meta.n_single
    if nd:
        _check(_lib.lightning_step(f32, _p(o), *head, _p(None), nd, H, D, V,
                                   _stream()), "lightning_step")
    if not meta.one_each:
        spans, chunks, seqs, base, n = _chunk_plan(
            meta, t.device,
            LIGHTNING_STEP_TOKENS if D <= LIGHTNING_MAX_D else 1 << 62)
        if spans is not None:
            _check(_lib.lightning_step(
                f32, _p(o), *head, _p(spans), spans.shape[0], H, D, V,
                _stream()), "lightning_step")
        if chunks is not None:
            scr = torch.empty(_lib.lightning_scratch(n, H, D, V),
                              dtype=dtype, device=t.device)
            _check(_lib.lightning_chunks(
                f32, _p(o), _p(scr), *head, _p(chunks), _p(seqs),
                seqs.shape[0], base, n, H, D, V, _stream()),
                "lightning_chunks")
    if w.per_head:
        return head_gate(o, w.norm, p, og, w.gate, dtype, H, V, w.eps, frag,
                         w.scale)
    if w.gate != "sigmoid" or w.norm is None or w.scale != 1.0:
        raise ValueError("norm over all heads: weight and sigmoid gate only")
    N = H * V
    if frag:
        res = _frag_rows(T, N, t)
        out = res.buf
    else:
        res = out = torch.empty((T, N), dtype=dtype, device=t.device)
    if T:
        _check(_lib.rms_gate(f32, _p(out), _p(o), _p(w.norm), *rows, og, T,
                             N, float(w.eps), int(frag), _stream()),
               "rms_gate")
    return res


def head_gate(o, norm, gate, og, act, dtype, H, V, eps, frag, mult=1.0):
    """Every head of mult * o [T, H*V] fp32 normed by itself, times the
    weight (shared [V], [H*V] or None) and the sigmoid or silu of the gate's
    columns og.."""
    T = o.shape[0]
    assert act in ("sigmoid", "silu") and _cols(gate) >= og + H * V \
        and (norm is None or norm.numel() in (V, H * V))
    if frag:
        res = _frag_rows(T, H * V, o)
        out = res.buf
    else:
        res = out = torch.empty((T, H * V), dtype=dtype, device=o.device)
    stride = V if norm is not None and norm.numel() == H * V else 0
    if T:
        _check(_lib.head_gate(
            int(dtype == torch.float32), _p(out), _p(o), float(mult),
            _p(norm), stride, *_rows(gate), og, int(act == "silu"), T, H, V,
            float(eps), int(frag), _stream()), "head_gate")
    return res


def pack_operand(w):
    """[N, K] as operands of 16 rows by 32 columns (lane = column group * 16
    + row, eight columns each) after one another; zeros fill up rows to 64
    and columns to 32."""
    N, K = w.shape
    w = torch.nn.functional.pad(w, (0, -K % 32, 0, -N % 64))
    return w.view(-1, 16, w.shape[1] // 32, 4, 8) \
        .permute(0, 2, 3, 1, 4).contiguous().view(-1)


DELTA_STEP_TOKENS = 4    # portions up to this walk token by token
DELTA_MAX_D = 256        # key width the chunk kernels take
DELTA_BYTES = 1 << 30    # chunk factors held at a time
CONV_STRIP = 16          # tokens of a portion that one wave convolves


def _chunk_groups(meta, dev, step_tokens, most):
    """The chunks of _chunk_plan in groups of about `most`, the sequences'
    chunks side by side: [(chunks, seqs)].  What a group needs in memory is
    used again by the next, and stays near."""
    key = f"_chunk_groups_{step_tokens}_{most}"
    groups = getattr(meta, key, None)
    if groups is None:
        _, chunks, seqs, _, _ = _chunk_plan(meta, dev, step_tokens)
        chunks, seqs = chunks.tolist(), seqs.tolist()
        longest = max(n for _, n in seqs)
        each = max(1, most // len(seqs))        # chunks of a sequence
        n = -(-longest // each)
        each = -(-longest // n)
        groups = []
        for lo in range(0, longest, each):
            c, s = [], []
            for first, count in seqs:
                part = chunks[first + lo:first + min(count, lo + each)] \
                    if lo < count else []
                if part:
                    s.append((len(c), len(part)))
                    c += part
            groups.append(tuple(torch.tensor(x, dtype=torch.int32).to(dev)
                                for x in (c, s)))
        setattr(meta, key, groups)
    return groups


def _conv_strips(meta, taps, dev):
    """Strips of the portions, int32 [n, 4]: first row, rows, the portion's
    first row and end.  No strip but a portion's first reads inputs from
    before the portion."""
    size = max(CONV_STRIP, taps - 1)
    key = f"_strips_{size}"
    t = getattr(meta, key, None)
    if t is None:
        strips, row = [], 0
        for n in meta.layout()[1]:
            strips += [(row + i, min(size, n - i), row, row + n)
                       for i in range(0, n, size)]
            row += n
        t = torch.tensor(strips, dtype=torch.int32).to(dev)
        setattr(meta, key, t)
    return t


class _HeadOut(NamedTuple):
    """The norm and gate behind a recurrence: weight, gate rows, the gate's
    first column, and the epsilon."""
    norm: torch.Tensor
    gate: torch.Tensor
    og: int
    eps: float


def _delta(gen, x, offsets, qs, ks, decay, beta, a_bias, state, G, slots, pos,
           meta, out: _HeadOut, frag):
    """The recurrence over prepared rows, norm and gate -> [T, H*V]."""
    H, D, V = state.shape[1:]
    T, dev, f32 = x.shape[0], x.device, _is_f32(x)
    assert state.dtype == torch.float32 and state.is_contiguous() \
        and x.stride(1) == 1 and out.gate.dtype == x.dtype \
        and out.gate.stride(1) == 1 and out.norm.numel() in (V, H * V) \
        and out.og + H * V <= out.gate.shape[1]
    head = (_p(x), x.stride(0), *offsets, _p(qs), _p(ks), ks.stride(0),
            _p(decay), _p(beta), _p(a_bias), _p(state), _p(slots), _p(pos))
    nd = meta.n_single
    stride = V if out.norm.numel() == H * V else 0

    def step(o, spans, n, whole):
        _check(_lib.delta_step(
            f32, gen, _p(o), *head, _p(spans), n, H, G, D, V, _p(out.norm),
            stride, _p(out.gate), out.gate.stride(0), out.og,
            float(out.eps), 2 if whole and frag else int(whole), _stream()),
            "delta_step")

    if meta.one_each and T and _lib.delta_whole(
            T, H, D, V, offsets[2], x.stride(0)):
        res = _frag_rows(T, H * V, x) if frag else \
            torch.empty((T, H * V), dtype=x.dtype, device=dev)
        step(res.buf if frag else res, None, T, True)
        return res
    o = torch.empty((T, H * V), dtype=torch.float32, device=dev)
    if nd:
        step(o, None, nd, False)
    if not meta.one_each:
        spans, chunks, seqs, _, _ = _chunk_plan(
            meta, dev, DELTA_STEP_TOKENS if D <= DELTA_MAX_D else 1 << 62)
        if spans is not None:
            step(o, spans, spans.shape[0], False)
        if chunks is not None:
            one = _lib.delta_scratch_floats(gen, 1, H, D)
            groups = _chunk_groups(meta, dev, DELTA_STEP_TOKENS,
                                   max(1, DELTA_BYTES // (4 * one)))
            scr = torch.empty(max(c.shape[0] for c, _ in groups) * one,
                              dtype=torch.float32, device=dev)
            for chunks, seqs in groups:
                _check(_lib.delta_chunks(
                    f32, gen, _p(o), _p(scr), *head, _p(chunks),
                    chunks.shape[0], _p(seqs), seqs.shape[0], H, G, D, V,
                    _stream()), "delta_chunks")
    return head_gate(o, out.norm, out.gate, out.og, "sigmoid", x.dtype, H, V,
                     out.eps, frag)


def gated_delta(p, w, state, conv_state, slot_ids, positions, meta, frag):
    H, G, D, V = w.heads, w.kv_heads, w.dim, w.vdim
    o_in, ob, oa, og = w.offsets
    taps, C = w.conv.shape
    ra, rg = w.a2.rank, w.g2.rank
    t = p.parts if isinstance(p, Partials) else p
    T, dev, dtype = t.shape[-2], t.device, w.a2.w.dtype
    assert C == 2 * G * D + H * V and state.shape[1:] == (H, D, V) \
        and conv_state.shape[1:] == (taps - 1, C) \
        and conv_state.dtype == torch.float32 \
        and conv_state.is_contiguous() and w.conv.is_contiguous() \
        and max(o_in + C, ob + H, oa + ra, og + rg) <= t.shape[-1] \
        and w.a2.w.shape[0] == w.dt_bias.numel() == H * D \
        and w.g2.w.shape[0] == H * V and w.rate.numel() == H \
        and w.norm.numel() == V
    assert isinstance(p, Partials) or p.dtype == dtype
    assert not frag or meta.one_each
    new = lambda *shape, dtype=torch.float32: torch.empty(
        shape, dtype=dtype, device=dev)
    y, gate = new(T, C, dtype=dtype), new(T, H * V, dtype=dtype)
    scales, decay, beta = new(T, 2 * G), new(T, H * D), new(T, H)
    slots, pos = _i32(slot_ids), _i32(positions)
    strips = None if meta.one_each else _conv_strips(meta, taps, dev)
    n = T if strips is None else strips.shape[0]
    if T:
        _check(_lib.gated_rows(
            int(dtype == torch.float32), *_rows(p), o_in, ob, oa, ra, og, rg,
            _p(w.conv), taps, _p(conv_state), _p(slots), _p(pos), _p(strips),
            n, _p(w.a2.packed), _p(w.rate), _p(w.dt_bias), _p(w.g2.packed),
            _p(y),
            _p(scales), _p(decay), _p(beta), _p(gate), T, H, G, D, V,
            _stream()), "gated_rows")
    return _delta(0, y, (0, G * D, 2 * G * D, 0), scales, scales[:, G:],
                  decay, beta, None, state, G, slots, pos, meta,
                  _HeadOut(w.norm, gate, 0, w.eps), frag)


def general_delta(p, w, state, slot_ids, positions, meta, frag):
    H, D = w.heads, w.dim
    o_r, ok, ov, oa, og, ow = w.offsets
    rank = w.w2.rank
    t = p.parts if isinstance(p, Partials) else p
    T, cols, dev, dtype = t.shape[-2], t.shape[-1], t.device, w.w2.w.dtype
    assert state.shape[1:] == (H, D, D) and w.w2.w.shape[0] == H * D \
        and max(w.offsets[:5]) + H * D <= cols \
        and ow + rank <= cols and w.w0.numel() == w.a_bias.numel() \
        == w.norm.numel() == H * D
    assert isinstance(p, Partials) or p.dtype == dtype
    assert not frag or meta.one_each
    scales = torch.empty((T, H), dtype=torch.float32, device=dev)
    decay = torch.empty((T, H * D), dtype=torch.float32, device=dev)
    whole = isinstance(p, Partials)
    y = torch.empty((T, cols), dtype=dtype, device=dev) if whole else p
    slots, pos = _i32(slot_ids), _i32(positions)
    if T:
        _check(_lib.general_rows(
            int(dtype == torch.float32), *_rows(p), ok, ow, rank,
            _p(w.w2.packed), _p(w.w0), _p(scales), _p(decay), _p(y if whole else None), cols,
            T, H, D, _stream()), "general_rows")
    return _delta(1, y, (o_r, ok, ov, oa), None, scales, decay, None,
                  w.a_bias, state, H, slots, pos, meta,
                  _HeadOut(w.norm, y, og, w.eps), frag)


# ---------------------------------------------------------------------------
# norms on sublayer outputs, sigmoid attention, mixture of experts

def rms_residual(x, y, post, pre, mult, eps, embed, tokens, embed_scale,
                 rows, need_x, frag, route=None, shift=None, tail=False,
                 bare=False):
    """route: MoeWeights whose router takes h on the way; then (x', h,
    (chosen, share))."""
    W = embed.shape[1]
    if x is not None:
        T = x.shape[0]
        assert x.dtype == torch.float32 and x.is_contiguous()
    elif bare:
        T = y.parts.shape[1] if isinstance(y, Partials) else y.shape[0]
    else:
        T = tokens.shape[0]
    assert not tail or tokens.shape[0] == T
    n_part, part_stride, row_stride, share = 1, 0, W, None
    yt = y
    if isinstance(y, Partials):
        yt, n_part, part_stride = y.parts, y.parts.shape[0], T * W
        assert yt.shape[1:] == (T, W)
    elif isinstance(y, Weighted):
        yt, share, n_part = y.parts, y.share, y.parts.shape[1]
        part_stride, row_stride = W, n_part * W
        assert yt.shape == (T, n_part, W) and share.shape == (T, n_part) \
            and share.is_contiguous() and share.dtype == torch.float32
    elif y is not None:
        assert y.shape == (T, W)
    assert yt is None or (yt.is_contiguous() and yt.dtype in
                          (embed.dtype, torch.float32))
    n = T if rows is None else rows.shape[0]
    HW = 2 * W if tail else W
    if frag:
        assert embed.dtype == torch.bfloat16 and W % 64 == 0
        res = _frag_rows(n, HW, embed)
        h = res.buf
    else:
        res = h = torch.empty((n, HW), dtype=embed.dtype, device=embed.device)
    x_out = torch.empty((n, W), dtype=torch.float32, device=embed.device) \
        if need_x else None
    chosen = route_share = None
    E = top = 0
    if route is not None:
        E, top = route.router.shape[0], route.top
        assert route.router.shape[1] == W and rows is None
        chosen = torch.empty((n, top), dtype=torch.int32, device=embed.device)
        route_share = torch.empty((n, top), dtype=torch.float32,
                                  device=embed.device)
    if n:
        _check(_lib.rms_residual(
            _is_f32(h), _p(x_out), _p(h), _p(x), _p(embed),
            _p(None if tokens is None else _i32(tokens)), float(embed_scale),
            _p(yt), int(yt is not None and yt.dtype == torch.float32),
            n_part, part_stride, row_stride, _p(share), _p(post), _p(pre),
            _p(shift), float(mult), float(eps), _p(rows), n, W, int(tail),
            int(bare), int(frag),
            _p(None if route is None else route.router), _p(chosen),
            _p(route_share), E, top, _stream()), "rms_residual")
    if route is not None:
        return x_out, res, (chosen, route_share)
    return x_out, res


def _src(y, T, W, dtype):
    """A sublayer's result, whole or in parts: (pointer, fp32?, parts,
    stride of a part)."""
    if y is None:
        return _p(None), 0, 1, 0
    t = y.parts if isinstance(y, Partials) else y
    assert t.is_contiguous() and t.shape[-2:] == (T, W) \
        and t.dtype in (dtype, torch.float32)
    return (_p(t), int(t.dtype == torch.float32),
            t.shape[0] if isinstance(y, Partials) else 1, T * W)


def ln_residual(x, y, norm, mult, eps, scale, embed, tokens, rows, need_x,
                frag, then):
    W, dtype = embed.shape[1], embed.dtype
    T = (tokens if x is None else x).shape[0]
    assert x is None or (x.dtype == torch.float32 and x.is_contiguous())
    pairs, share = ((y, None),), 1.0
    if isinstance(y, Branches):
        pairs, share = y.pairs, y.share
        if not 1 <= len(pairs) <= 2:
            raise ValueError(f"{len(pairs)} branches: no kernel")
    pairs = tuple(pairs) + ((None, None),) * (2 - len(pairs))
    n = T if rows is None else rows.shape[0]
    if frag:
        assert dtype == torch.bfloat16 and W % 64 == 0
        res = _frag_rows(n, W, embed)
        h = res.buf
    else:
        res = h = torch.empty((n, W), dtype=dtype, device=embed.device)
    if x is not None and y is None and rows is None:
        x_out, write = x, None               # nothing to add
    else:
        x_out = write = torch.empty(
            (n, W), dtype=torch.float32, device=embed.device) \
            if need_x else None
    nw, nb = norm if norm is not None else (None, None)
    tw, tb = then if then is not None else (None, None)
    if n:
        _check(_lib.ln_residual(
            _is_f32(h), _p(write), _p(h), _p(x), _p(embed),
            _p(None if tokens is None else _i32(tokens)),
            *_src(pairs[0][0], T, W, dtype), *_src(pairs[1][0], T, W, dtype),
            _p(pairs[0][1]), _p(pairs[1][1]), float(share), _p(scale), _p(nw),
            _p(nb), float(mult), _p(tw), _p(tb), float(eps), _p(rows), n, W,
            int(frag), _stream()), "ln_residual")
    return x_out, res


ROUTE_FUSED_MAX = 16      # experts the row kernel takes along


def rms_residual_route(x, y, post, mult, eps, moe, embed, tokens,
                       embed_scale, frag):
    args = (x, y, post, None, mult, eps, embed, tokens, embed_scale, None,
            True, frag)
    if frag and moe.router.shape[0] <= ROUTE_FUSED_MAX:
        return rms_residual(*args, route=moe)
    x, h = rms_residual(*args)
    return x, h, moe_route(h, moe)


def qk_norm_append(p, cache, run, w, q_norm, k_norm, eps, slot_ids,
                   positions):
    kp, vp = cache.key_pool[run], cache.value_pool[run]
    H, G, D, V = w.heads, w.kv_heads, w.dim, w.vdim
    if isinstance(p, Partials):
        p, n_part, part_stride = p.parts, p.parts.shape[0], p.parts.stride(0)
        T, row_stride = p.shape[1], p.stride(1)
    else:
        n_part, part_stride, T, row_stride = 1, 0, p.shape[0], p.stride(0)
    assert p.stride(-1) == 1 and p.shape[-1] >= H * D + G * (D + V) \
        and p.dtype in (kp.dtype, torch.float32)
    assert kp.shape[1:3] == (G, cache.page_size) and kp.shape[3] >= D \
        and vp.shape[3] >= V and q_norm.numel() == H * D \
        and k_norm.numel() == G * D
    q = torch.empty((T, H, kp.shape[3]), dtype=kp.dtype, device=kp.device)
    if T:
        _check(_lib.qk_norm_append(
            _is_f32(q), _p(q), _p(kp), _p(vp), _p(p),
            int(p.dtype == torch.float32), n_part, part_stride, row_stride,
            _p(q_norm), _p(k_norm), _p(_i32(slot_ids)), _p(_i32(positions)),
            _p(cache.page_table), T, H, G, D, V, kp.shape[3], vp.shape[3],
            cache.page_size, cache.page_table.shape[1], float(eps),
            _stream()), "qk_norm_append")
    return q


ATTN_MAX = 256         # key and value widths
ATTN_SHORT = 8         # portions up to this many tokens split the context
ATTN_SPLIT_MAX = 16
ATTN_LARGE = 128 * 1024   # (token, head) rows from which tiles are large:
                             # they share staged keys, small ones share load


def _tile_plan(meta, R, rows, dev):
    """Tiles of one attention shape: leading single tokens and short
    portions in 16-row tiles for the context-splitting kernel, the rest in
    `rows`-row tiles."""
    key = f"_tiles_{R}_{rows}"
    plan = getattr(meta, key, None)
    if plan is not None:
        return plan
    _, q_lens, kv_lens = meta.layout()
    i = row = kv = 0
    short, long_ = [], []
    while i < len(q_lens) and q_lens[i] <= ATTN_SHORT:
        lo, hi = row * R, (row + q_lens[i]) * R
        short += [(r, min(16, hi - r)) for r in range(lo, hi, 16)]
        kv = max(kv, kv_lens[i])
        row += q_lens[i]
        i += 1
    n_short = row
    for n in q_lens[i:]:
        lo, hi = row * R, (row + n) * R
        long_ += [(r, min(rows, hi - r)) for r in range(lo, hi, rows)]
        row += n
    t32 = lambda x: torch.tensor(x, dtype=torch.int32).to(dev) \
        if x else None
    plan = (t32(short), n_short, kv, t32(long_))
    setattr(meta, key, plan)
    return plan


def sigmoid_attention(q, cache, run, w, slot_ids, positions, meta, frag):
    T, H, Dp = q.shape
    kp, vp = cache.key_pool[run], cache.value_pool[run]
    G, V, R = w.kv_heads, w.vdim, w.heads // w.kv_heads
    f32 = _is_f32(q)
    if max(Dp, vp.shape[3]) > ATTN_MAX:
        raise ValueError(f"sigmoid attention with head widths {w.dim}/"
                         f"{w.vdim}: no kernel")
    assert q.is_contiguous() and kp.dtype == q.dtype \
        and kp.shape[1:] == (G, cache.page_size, Dp) and H == w.heads \
        and w.decay.numel() == w.reach.numel() == w.bias.numel() == H
    assert not frag or meta.one_each
    if frag:
        res = _frag_rows(T, H * V, q)
        out = res.buf
    else:
        res = out = torch.empty((T, H * V), dtype=q.dtype, device=q.device)
    if meta.one_each:
        n_items, n_tok, kv = T * -(-R // 16), T, meta.max_kv
        short = long_ = None
    else:
        rows = _lib.sigmoid_rows(f32, Dp, vp.shape[3]) \
            if T * H >= ATTN_LARGE else 64
        short, n_tok, kv, long_ = _tile_plan(meta, R, rows, q.device)
        n_items = 0 if short is None else short.shape[0]

    def launch(item_rows, items, n, t0, tokens, split, part):
        _check(_lib.sigmoid_attn(
            f32, item_rows, _p(out), _p(part), _p(q), _p(kp), _p(vp),
            _p(cache.page_table), _p(_i32(slot_ids)), _p(_i32(positions)),
            _p(items), n, t0, tokens, T, H, G, V, Dp, vp.shape[3],
            cache.page_size, cache.page_table.shape[1], split, int(frag),
            w.scale, w.softcap, _p(w.decay), _p(w.reach), _p(w.bias),
            w.window, _stream()), "sigmoid_attn")

    if n_items:
        seen = min(kv, w.window) if w.window else kv
        split = max(1, min(256 // (n_items * G),
                           -(-seen // _lib.sigmoid_step(f32)),
                           ATTN_SPLIT_MAX))
        part = torch.empty((split, T, H * V), dtype=torch.float32,
                           device=q.device) if split > 1 else None
        launch(16, short, n_items, 0, n_tok, split, part)
    if long_ is not None:
        launch(rows, long_, long_.shape[0], 0, T, 1, None)
    return res


def rope_qkv_append(p, bias, cache, run, w, rope, slot_ids, positions):
    kp, vp = cache.key_pool[run], cache.value_pool[run]
    H, G, D, V = w.heads, w.kv_heads, w.dim, w.vdim
    T, n = slot_ids.shape[0], H * D + G * (D + V)
    assert _cols(p) >= n and (bias is None or bias.numel() >= n)
    assert kp.shape[1:3] == (G, cache.page_size) and kp.shape[3] >= D \
        and vp.shape[3] >= V and rope.dims <= D
    assert not rope.dims or (rope.table.shape[1] == rope.dims
                             and rope.table.shape[0] >= cache.max_ctx)
    if rope.halves:
        raise ValueError("rotation by halves without head norms: no kernel")
    q = torch.empty((T, H, kp.shape[3]), dtype=kp.dtype, device=kp.device)
    rows = _rows(p)
    assert rows[1] or kp.dtype == torch.bfloat16
    if T:
        _check(_lib.rope_qkv_append(
            _is_f32(q), _p(q), _p(kp), _p(vp), *rows, _p(bias),
            _p(rope.table), rope.dims, _p(_i32(slot_ids)),
            _p(_i32(positions)), _p(cache.page_table), T, H, G, D, V,
            kp.shape[3], vp.shape[3], cache.page_size,
            cache.page_table.shape[1], _stream()), "rope_qkv_append")
    return q


def qkv_norm_rope_append(p, norms, cache, run, w, rope, slot_ids, positions):
    kp, vp = cache.key_pool[run], cache.value_pool[run]
    H, G, D, V = w.heads, w.kv_heads, w.dim, w.vdim
    T = slot_ids.shape[0]
    if max(kp.shape[3], vp.shape[3]) > ATTN_MAX:
        raise ValueError(f"softmax attention with head widths {D}/{V}: no "
                         "kernel")
    if rope.dims and not rope.halves:
        raise ValueError("head norms with interleaved rotation: no kernel")
    assert _cols(p) >= H * D + G * (D + V) and norms.q.numel() == D \
        and norms.k.numel() == D \
        and (norms.gain is None or norms.gain.numel() == H)
    assert kp.shape[1:3] == (G, cache.page_size) and kp.shape[3] >= D \
        and vp.shape[3] >= V and rope.dims <= D
    assert not rope.dims or (rope.table.shape[1] == rope.dims
                             and rope.table.shape[0] >= cache.max_ctx)
    q = torch.empty((T, H, kp.shape[3]), dtype=kp.dtype, device=kp.device)
    rows = _rows(p)
    assert rows[1] or kp.dtype == torch.bfloat16
    if T:
        _check(_lib.qkv_norm_rope(
            _is_f32(q), _p(q), _p(kp), _p(vp), *rows, _p(norms.q),
            _p(norms.k), _p(norms.gain), int(norms.values), float(norms.eps),
            _p(rope.table), rope.dims, _p(_i32(slot_ids)),
            _p(_i32(positions)), _p(cache.page_table), T, H, G, D, V,
            kp.shape[3], vp.shape[3], cache.page_size,
            cache.page_table.shape[1], _stream()), "qkv_norm_rope")
    return q


def softmax_attention(q, cache, run, w, slot_ids, positions, meta, frag,
                      gate=None):
    T, H, Dp = q.shape
    kp, vp = cache.key_pool[run], cache.value_pool[run]
    G, V, R = w.kv_heads, w.vdim, w.heads // w.kv_heads
    Vp, f32 = vp.shape[3], _is_f32(q)
    if max(Dp, Vp) > ATTN_MAX:
        raise ValueError(f"softmax attention with head widths {w.dim}/"
                         f"{w.vdim}: no kernel")
    assert q.is_contiguous() and kp.dtype == q.dtype \
        and kp.shape[1:] == (G, cache.page_size, Dp) and H == w.heads \
        and (w.sink is None or w.sink.numel() == H)
    gp, og = (None, 0) if gate is None else gate
    assert gp is None or og + H <= _cols(gp)
    assert not frag or meta.one_each
    if frag:
        res = _frag_rows(T, H * V, q)
        out = res.buf
    else:
        res = out = torch.empty((T, H * V), dtype=q.dtype, device=q.device)
    if meta.one_each:
        n_items, n_tok, kv = T * -(-R // 16), T, meta.max_kv
        short = long_ = None
    else:
        rows = _lib.softmax_rows(f32, Dp, Vp) if T * H >= ATTN_LARGE else 64
        short, n_tok, kv, long_ = _tile_plan(meta, R, rows, q.device)
        n_items = 0 if short is None else short.shape[0]

    def launch(item_rows, items, n, tokens, split, part, ml):
        _check(_lib.softmax_attn(
            f32, item_rows, _p(out), _p(part), _p(ml), _p(q), _p(kp), _p(vp),
            _p(cache.page_table), _p(_i32(slot_ids)), _p(_i32(positions)),
            _p(items), n, 0, tokens, T, H, G, V, Dp, Vp, cache.page_size,
            cache.page_table.shape[1], split, int(frag), w.scale, _p(w.sink),
            w.window, w.chunk, *_rows(gp), og, _stream()), "softmax_attn")

    if n_items:
        seen = w.reach(kv)
        split = max(1, min(256 // (n_items * G),
                           -(-seen // _lib.softmax_step(f32)),
                           ATTN_SPLIT_MAX))
        part = ml = None
        if split > 1:
            part = torch.empty((split, T, H * V), dtype=torch.float32,
                               device=q.device)
            ml = torch.empty((split, T, H, 2), dtype=torch.float32,
                             device=q.device)
        launch(16, short, n_items, n_tok, split, part, ml)
    if long_ is not None:
        launch(rows, long_, long_.shape[0], T, 1, None, None)
    return res


def moe_route(h, w):
    frag = isinstance(h, FragRows)
    E, K = w.router.shape
    T = h.rows if frag else h.shape[0]
    x = h.buf if frag else h
    assert frag or (h.shape[1] == K and h.is_contiguous()
                    and h.dtype == w.router.dtype)
    dev = w.router.device
    chosen = torch.empty((T, w.top), dtype=torch.int32, device=dev)
    share = torch.empty((T, w.top), dtype=torch.float32, device=dev)
    if T:
        _check(_lib.moe_route(_is_f32(w.router), _p(chosen), _p(share),
                              _p(x), _p(w.router), T, K, E, w.top, int(frag),
                              _stream()), "moe_route")
    return chosen, share


def moe_experts(h, w, chosen, share, packs):
    E, F2, K = w.gate_up.shape
    N, F = w.down.shape[1:]
    T, top = chosen.shape
    A = T * top
    dev = w.router.device
    if isinstance(h, FragRows):
        act = _frag_rows(A, F, w.router)
        out = torch.empty((T, top, N), dtype=torch.float32, device=dev)
        for gu, x, pk, n, k in ((1, h.buf, packs["gate_up"], F2, K),
                                (0, act.buf, packs["down"], N, F)):
            _check(_lib.moe_stream(gu, _p(act.buf), _p(out), _p(x), _p(pk),
                                   _p(chosen), A, top, E, n, k, _stream()),
                   "moe_stream")
        return Weighted(out, share)
    f32 = _is_f32(w.router)
    out = torch.empty((T, top, N), dtype=w.router.dtype, device=dev)
    if T == 0:
        return Weighted(out, share)
    fast = not f32 and K % 64 == 0 and N % 4 == 0 and A >= 64
    TM = 128 if fast else 16
    # an expert without tokens has no tile
    n_tiles = A // TM + min(E, A)
    tile_e = torch.empty(n_tiles, dtype=torch.int32, device=dev)
    perm = torch.empty(n_tiles * TM, dtype=torch.int32, device=dev)
    _check(_lib.moe_plan(_p(tile_e), _p(perm), _p(chosen), A, E, TM, n_tiles,
                         _stream()), "moe_plan")
    act = torch.empty((n_tiles * TM, F), dtype=w.router.dtype, device=dev)
    for gu, o, x, m, n, k in ((1, act, h, "gate_up", F2, K),
                              (0, out, act, "down", N, F)):
        pk, m = packs.get(m), getattr(w, m)
        if fast and pk is not None:
            _check(_lib.moe_gemm_packed(
                gu, _p(o), _p(x), _p(pk), _p(tile_e), _p(perm), n_tiles, top,
                n, k, _stream()), "moe_gemm_packed")
        elif fast:
            _check(_lib.moe_gemm(gu, _p(o), _p(x), _p(m), _p(tile_e),
                                 _p(perm), n_tiles, top, n, k, _stream()),
                   "moe_gemm")
        else:
            _check(_lib.moe_mm(f32, gu, _p(o), _p(x), _p(m), _p(tile_e),
                               _p(perm), n_tiles, top, n, k, _stream()),
                   "moe_mm")
    return Weighted(out, share)


def sample_gumbel(logits, temps, seeds, ctrs, noise=None, out=None):
    """Exact temperature sampling (Gumbel-max): token ~ softmax(l/T) per
    row; rows with temps<=0 are greedy argmax.  Counter-based noise from
    (seeds[row], ctrs[row], v) — graph-replay-safe and reproducible per
    request.  noise: optional [B,V] uniform(0,1) override (tests)."""
    B, V = logits.shape
    l = logits if logits.dtype == torch.bfloat16 else logits.bfloat16()
    if out is None:
        out = torch.empty(B, dtype=torch.int32, device=logits.device)
    sp = min(32, max(1, 768 // max(1, B)))
    pb = pi = ctypes.c_void_p(0)
    if sp > 1:
        key = ("gmb", B, sp, str(logits.device))
        t = _scratch.get(key)
        if t is None:
            t = (torch.empty(B * sp, dtype=torch.float32,
                             device=logits.device),
                 torch.empty(B * sp, dtype=torch.int32,
                             device=logits.device))
            _scratch[key] = t
        pb, pi = _p(t[0]), _p(t[1])
    _check(_lib.sample_gumbel_bf16(
        _p(out), _p(l), _p(temps), _p(seeds), _p(ctrs), _p(noise),
        B, V, pb, pi, sp, _stream()), "sample_gumbel")
    return out


def sample(logits, temperature, top_k, top_p, generator=None):
    if torch.is_tensor(temperature):
        all_greedy = bool((temperature <= 0).all())
    else:
        all_greedy = temperature <= 0
    if all_greedy:
        B, V = logits.shape
        if V % 8 or not logits.is_contiguous():
            return logits.argmax(-1)     # rows not aligned for the kernel
        out = torch.empty(B, dtype=torch.int32, device=logits.device)
        f32 = logits.dtype == torch.float32
        l = logits if f32 or logits.dtype == torch.bfloat16 \
            else logits.bfloat16()
        # split-V: B blocks alone underfill the chip at decode batch sizes
        sp = min(32, max(1, 768 // max(1, B)))
        pb = pi = ctypes.c_void_p(0)
        if sp > 1:
            key = ("amax", B, sp, str(logits.device))
            t = _scratch.get(key)
            if t is None:
                t = (torch.empty(B * sp, dtype=torch.float32,
                                 device=logits.device),
                     torch.empty(B * sp, dtype=torch.int32,
                                 device=logits.device))
                _scratch[key] = t
            pb, pi = _p(t[0]), _p(t[1])
        fn = _lib.argmax_f32 if f32 else _lib.argmax_bf16
        _check(fn(_p(out), _p(l), B, V, pb, pi, sp, _stream()), "argmax")
        return out.long()
    # stochastic host path.  When every stochastic row carries
    # 0 < top_k <= 256 the sampling is EXACT over the top-256 candidates
    # (its nucleus is a subset of its top-k; probabilities use a
    # full-vocabulary logsumexp, so the top-p mass cut is the true one)
    # and costs a topk + tiny multinomial instead of the full-vocab sort
    # (~0.5 ms/step at V=128256).  Anything else falls back to the
    # fp32 reference (exact, sort-based).
    B, V = logits.shape
    dev = logits.device
    if not torch.is_tensor(temperature):
        temperature = torch.full((B,), float(temperature), device=dev)
    tk = top_k if torch.is_tensor(top_k) else torch.full(
        (B,), int(top_k or 0), dtype=torch.long, device=dev)
    tp = top_p if torch.is_tensor(top_p) else torch.full(
        (B,), float(top_p if top_p else 1.0), device=dev)
    tk = tk.long()
    stoch = temperature > 0
    C = min(256, V)
    capped_ok = bool(((tk > 0) & (tk <= C) | ~stoch).all())
    if not capped_ok:
        return ref.sample(logits, temperature, tk, tp, generator)
    l = logits.float()
    t = torch.where(stoch, temperature, torch.ones_like(temperature))
    lt = l / t.unsqueeze(1)
    v, idx = torch.topk(lt, C, dim=-1)
    lse = torch.logsumexp(lt, dim=-1, keepdim=True)
    p = torch.exp(v - lse)                      # exact full-vocab probs
    ar = torch.arange(C, device=dev)
    keep = ar.unsqueeze(0) < tk.clamp(min=1, max=C).unsqueeze(1)
    cum = p.cumsum(dim=-1)
    keep &= (cum - p) < tp.unsqueeze(1)
    keep[:, 0] = True
    pm = p * keep
    pick = torch.multinomial(pm / pm.sum(-1, keepdim=True), 1,
                             generator=generator).squeeze(1)
    out_s = idx.gather(1, pick.unsqueeze(1)).squeeze(1)
    if bool(stoch.all()):
        return out_s
    # greedy rows override with the true argmax
    return torch.where(stoch, out_s, l.argmax(-1))


def decode_pure(cache, layer, meta, split, chunk=64):
    """Staging-only diagnostic for decode attention (see decode_attn.hip
    k_decode_pure)."""
    sink = torch.zeros(1, dtype=torch.float32, device=cache.k_pool.device)
    kp, vp = _layer_ptrs(cache, layer)
    S = meta.slot_ids.shape[0]
    _check(_lib.decode_pure_bf16(
        _p(sink), kp, vp, _p(cache.page_table), _p(meta.slot_ids.int()),
        _p(meta.seq_lens.int()), S, cache.n_kv_heads, cache.page_size,
        cache.page_table.shape[1], split, chunk, _stream()),
        "decode_pure")
    return sink
