// Shared pieces of the kernels that run in bf16 and in true fp32: typed
// loads and stores, wave reductions, and a 16x16 matrix-core tile whose
// fragments look the same for both types.
#pragma once
#include <hip/hip_runtime.h>
#include <hip/hip_bf16.h>
#include <cstdint>

typedef __hip_bfloat16 bf16;
typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) __bf16 bf16x4;
typedef __attribute__((ext_vector_type(4))) float f32x4;

#define DEV static __device__ __forceinline__

DEV float ldf(const float* p) { return *p; }
DEV float ldf(const bf16* p) { return __bfloat162float(*p); }
DEV void stf(float* p, float v) { *p = v; }
DEV void stf(bf16* p, float v) { *p = __float2bfloat16(v); }

// VEC consecutive elements as floats; VEC is 1, 4 or 8 and the address is
// aligned to VEC elements
template <int VEC>
DEV void ldv(const float* p, float* o) {
    if constexpr (VEC == 1) o[0] = *p;
    else {
        #pragma unroll
        for (int i = 0; i < VEC; i += 4) {
            const f32x4 v = *reinterpret_cast<const f32x4*>(p + i);
            o[i] = v[0]; o[i + 1] = v[1]; o[i + 2] = v[2]; o[i + 3] = v[3];
        }
    }
}
template <int VEC>
DEV void ldv(const bf16* p, float* o) {
    if constexpr (VEC == 1) o[0] = __bfloat162float(*p);
    else if constexpr (VEC == 4) {
        const bf16x4 v = *reinterpret_cast<const bf16x4*>(p);
        #pragma unroll
        for (int i = 0; i < 4; i++) o[i] = (float)v[i];
    } else {
        const bf16x8 v = *reinterpret_cast<const bf16x8*>(p);
        #pragma unroll
        for (int i = 0; i < 8; i++) o[i] = (float)v[i];
    }
}
template <int VEC>
DEV void stv(float* p, const float* o) {
    if constexpr (VEC == 1) *p = o[0];
    else {
        #pragma unroll
        for (int i = 0; i < VEC; i += 4)
            *reinterpret_cast<f32x4*>(p + i) =
                f32x4{o[i], o[i + 1], o[i + 2], o[i + 3]};
    }
}
template <int VEC>
DEV void stv(bf16* p, const float* o) {
    if constexpr (VEC == 1) *p = __float2bfloat16(o[0]);
    else if constexpr (VEC == 4) {
        bf16x4 v;
        #pragma unroll
        for (int i = 0; i < 4; i++) v[i] = (__bf16)o[i];
        *reinterpret_cast<bf16x4*>(p) = v;
    } else {
        bf16x8 v;
        #pragma unroll
        for (int i = 0; i < 8; i++) v[i] = (__bf16)o[i];
        *reinterpret_cast<bf16x8*>(p) = v;
    }
}

// Rows of a matrix that may still be the partial sums of a split product:
// n_part of them part_stride apart, rows ld apart.
template <typename P> struct Rows {
    const P* p;
    int n_part;
    int64_t part_stride, ld;
};
// VEC columns of row t from column c on
template <int VEC, typename P>
DEV void ldrow(const Rows<P>& r, int64_t t, int c, float* v) {
    const P* p = r.p + t * r.ld + c;
    ldv<VEC>(p, v);
    int s = 1;
    for (; s + 1 < r.n_part; s += 2) {      // two at a time: half the waits
        float u[VEC], w[VEC];
        ldv<VEC>(p + s * r.part_stride, u);
        ldv<VEC>(p + (s + 1) * r.part_stride, w);
        #pragma unroll
        for (int i = 0; i < VEC; i++) v[i] = v[i] + u[i] + w[i];
    }
    if (s < r.n_part) {
        float u[VEC];
        ldv<VEC>(p + s * r.part_stride, u);
        #pragma unroll
        for (int i = 0; i < VEC; i++) v[i] += u[i];
    }
}

template <typename T> DEV float exp_of(float x) {
    if constexpr (sizeof(T) == 4) return expf(x);
    else return __expf(x);
}
template <typename T> DEV float sigmoid_of(float x) {
    if constexpr (sizeof(T) == 4) return 1.f / (1.f + expf(-x));
    else return __builtin_amdgcn_rcpf(1.f + __expf(-x));
}

template <typename T> DEV float silu_of(float x) {
    return x * sigmoid_of<T>(x);
}

// Activation-fragment layout ("frag"): the SAME MFMA fragment order the
// weight packs use, applied to a [32, K] activation: element (m, k) with
// k = b*64 + j*16 + h*8 + e lives at 16-byte unit ((b*4 + j)*64 + h*32
// + m), elem e.  Producers (GEMM epilogues, decode-attention combine,
// the embedding fragify kernel) write it; consumers stream it LINEARLY
// exactly like packed weights — the per-iteration x machinery (32-line
// scattered loads or LDS staging, measured 15-30% on top of the pure
// stream) disappears.  Buffers are always 32 rows; rows >= M hold
// garbage that MFMA carries in dead accumulator rows (never stored).
DEV int64_t frag_off(int m, int kcol) {
    const int b = kcol >> 6, j = (kcol >> 4) & 3, h = (kcol >> 3) & 1;
    return ((((int64_t)b * 4 + j) * 64) + h * 32 + m) * 8 + (kcol & 7);
}
// row r of a batch of up to 64: two halves of 32 rows, `cols` wide
DEV int64_t frag_row_off(int r, int c, int cols) {
    return (int64_t)(r >> 5) * 32 * cols + frag_off(r & 31, c);
}

DEV float wave_sum(float x) {
    #pragma unroll
    for (int o = 32; o; o >>= 1) x += __shfl_xor(x, o, 64);
    return x;
}
DEV float wave_max(float x) {
    #pragma unroll
    for (int o = 32; o; o >>= 1) x = fmaxf(x, __shfl_xor(x, o, 64));
    return x;
}

// Barrier for what goes through LDS: loads and stores to memory stay in
// flight across it.
DEV void lds_barrier() {
    asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
}

// sum over the block; every thread gets it.  s: one float per wave
template <int BS> DEV float block_sum(float v, float* s) {
    v = wave_sum(v);
    const int wid = threadIdx.x >> 6;
    if ((threadIdx.x & 63) == 0) s[wid] = v;
    __syncthreads();
    float t = 0.f;
    #pragma unroll
    for (int i = 0; i < BS / 64; i++) t += s[i];
    return t;
}

// odd series, relative error below 4e-7 up to 0.25
DEV float tanh_small(float x) {
    const float x2 = x * x;
    return x * (1.f + x2 * (-1.f / 3.f + x2 * (2.f / 15.f
                + x2 * (-17.f / 315.f))));
}
DEV float tanh_fast(float x) {
    const float a = fabsf(x);
    const float e = __expf(-2.f * a);
    const float big = copysignf((1.f - e) * __builtin_amdgcn_rcpf(1.f + e),
                                x);
    return a < 0.25f ? tanh_small(x) : big;
}
template <typename T> DEV float tanh_of(float x) {
    if constexpr (sizeof(T) == 4) return tanhf(x);
    else return tanh_fast(x);
}

// ---- 16x16 tile, 32 deep -------------------------------------------------
// A lane holds 8 elements of one row (A) or column (B): row/col = lane & 15,
// k = (lane >> 4) * 8 + e.  bf16 is one mfma_16x16x32; fp32 is eight
// mfma_16x16x4, one per element e: each takes k = {(lane >> 4) * 8 + e},
// and over all e the 32 k's are covered once.  Any other assignment of k to
// (lane group, e) gives the same product as long as A and B share it.
// The result: col = lane & 15, row = (lane >> 4) * 4 + i.
template <typename T> struct FragOf;
template <> struct FragOf<bf16> { typedef bf16x8 type; };
struct f32x8s { f32x4 lo, hi; };
template <> struct FragOf<float> { typedef f32x8s type; };
template <typename T> using Frag = typename FragOf<T>::type;

DEV f32x4 mma(bf16x8 a, bf16x8 b, f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}
DEV f32x4 mma(const f32x8s& a, const f32x8s& b, f32x4 c) {
    #pragma unroll
    for (int e = 0; e < 4; e++)
        c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.lo[e], b.lo[e], c, 0, 0, 0);
    #pragma unroll
    for (int e = 0; e < 4; e++)
        c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.hi[e], b.hi[e], c, 0, 0, 0);
    return c;
}

DEV bf16x8 frag8(const bf16* p) { return *reinterpret_cast<const bf16x8*>(p); }
DEV f32x8s frag8(const float* p) {
    return {*reinterpret_cast<const f32x4*>(p),
            *reinterpret_cast<const f32x4*>(p + 4)};
}
// two runs of four
DEV bf16x8 frag44(const bf16* p, const bf16* q) {
    const bf16x4 a = *reinterpret_cast<const bf16x4*>(p);
    const bf16x4 b = *reinterpret_cast<const bf16x4*>(q);
    return __builtin_shufflevector(a, b, 0, 1, 2, 3, 4, 5, 6, 7);
}
DEV f32x8s frag44(const float* p, const float* q) {
    return {*reinterpret_cast<const f32x4*>(p),
            *reinterpret_cast<const f32x4*>(q)};
}
DEV void frag_set(bf16x8& f, int e, float v) { f[e] = (__bf16)v; }
DEV void frag_set(f32x8s& f, int e, float v) {
    if (e < 4) f.lo[e] = v; else f.hi[e - 4] = v;
}
DEV float frag_get(const bf16x8& f, int e) { return (float)f[e]; }
DEV float frag_get(const f32x8s& f, int e) {
    return e < 4 ? f.lo[e] : f.hi[e - 4];
}
// an fp32 value as matrix operand: two bf16 terms, or itself
template <typename T> struct Terms;
template <> struct Terms<bf16> {
    static constexpr int N = 2;
    static DEV void split(float x, bf16* t) {
        t[0] = __float2bfloat16(x);
        t[1] = __float2bfloat16(x - __bfloat162float(t[0]));
    }
};
template <> struct Terms<float> {
    static constexpr int N = 1;
    static DEV void split(float x, float* t) { t[0] = x; }
};

// elements e with k0 + e < K; the rest are zero
template <typename T>
DEV Frag<T> frag_guard(const T* p, int k0, int K) {
    Frag<T> f;
    #pragma unroll
    for (int e = 0; e < 8; e++)
        frag_set(f, e, k0 + e < K ? ldf(p + k0 + e) : 0.f);
    return f;
}
template <typename T> DEV Frag<T> frag_zero() {
    Frag<T> f;
    #pragma unroll
    for (int e = 0; e < 8; e++) frag_set(f, e, 0.f);
    return f;
}

// ---- LDS transpose load (bf16) --------------------------------------------
typedef __attribute__((ext_vector_type(4))) short s16x4;
typedef __attribute__((ext_vector_type(8))) short s16x8;
typedef __attribute__((address_space(3))) s16x4 lds_s16x4;

// lane (lr, g) <- column c0 + lr of rows r0 + 4g .. +3, 16 columns of a tile
DEV s16x4 tr_read(const bf16* tile, int stride, int lane) {
    const int lr = lane & 15, g = lane >> 4;
    const bf16* p = tile + (4 * g + (lr >> 2)) * stride + (lr & 3) * 4;
    return __builtin_amdgcn_ds_read_tr16_b64_v4i16(
        (lds_s16x4*)const_cast<bf16*>(p));
}

// Operand of a product over the rows of an LDS tile: column lr of 32 rows,
// rows 4g + i of its two halves -- the order in which a 16x16 result holds
// its rows, so that the result of one product is an operand of the next.
DEV bf16x8 value_frag(const bf16* tile, int stride, int lane) {
    const s16x4 a = tr_read(tile, stride, lane);
    const s16x4 b = tr_read(tile + 16 * stride, stride, lane);
    return __builtin_bit_cast(
        bf16x8, __builtin_shufflevector(a, b, 0, 1, 2, 3, 4, 5, 6, 7));
}
DEV f32x8s value_frag(const float* tile, int stride, int lane) {
    const float* p = tile + (lane >> 4) * 4 * stride + (lane & 15);
    f32x8s f;
    #pragma unroll
    for (int e = 0; e < 4; e++) {
        f.lo[e] = p[e * stride];
        f.hi[e] = p[(16 + e) * stride];
    }
    return f;
}
// and that operand from two results
template <typename T> DEV Frag<T> weight_frag(const f32x4* s) {
    Frag<T> b;
    #pragma unroll
    for (int e = 0; e < 4; e++) {
        frag_set(b, e, s[0][e]);
        frag_set(b, e + 4, s[1][e]);
    }
    return b;
}

// zero the weights of keys a query does not see; s[j][i] is the key
// j * 16 + i after that of s[0][0], which is dist0 tokens back
template <int N>
DEV void mask_keys(f32x4* s, int dist0, int window) {
    #pragma unroll
    for (int j = 0; j < N; j++)
        #pragma unroll
        for (int i = 0; i < 4; i++) {
            const int d = dist0 - j * 16 - i;
            if (d < 0 || (window > 0 && d >= window)) s[j][i] = 0.f;
        }
}

// four columns c0.. of head h of token t; V values per head
template <typename T>
DEV void put_out(T* out, int t, int h, int c0, int H, int V, f32x4 v,
                 bool frag) {
    if (c0 >= V) return;
    const int c = h * V + c0;
    T* dst = out + (frag ? frag_row_off(t, c, H * V)
                         : (int64_t)t * H * V + c);
    float f[4] = {v[0], v[1], v[2], v[3]};
    if (V % 4 == 0) stv<4>(dst, f);
    else
        #pragma unroll
        for (int i = 0; i < 4; i++)
            if (c0 + i < V) stf(dst + i, f[i]);
}
