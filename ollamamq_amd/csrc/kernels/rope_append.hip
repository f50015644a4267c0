// gfx950 split of a fused attention projection with rotary positions, and
// the append to the paged pools.
//
// A token's pair (2i, 2i + 1) of a head's first `dims` dimensions is turned
// by the (cos, sin) at table[position][i]; whatever scales the rotation is in
// the table.  The projection may still be the partial sums of a split
// product.
//
// * k_rope_qkv_append: queries, keys and values with biases; rows of the
//   queries and of the pools are filled up to whole 16-byte vectors;
// * k_qkv_norm_rope: the same with every head normed by itself and pairs
//   (i, i + dims/2) turned;
// * k_latent_rope_append: queries whose heads end in a rotated part, the
//   normed latent and the one rotated key part that all heads share.
#include "tile_mma.h"

// VEC columns from dimension d of a head on, `far` their neighbours if VEC
// is 1; cs: the position's row of the table
template <int VEC>
DEV void turn(float* v, float far, int d, int dims, const float* cs) {
    if constexpr (VEC == 1) {
        if (d >= dims) return;
        const float c = cs[d & ~1], s = cs[d | 1];
        v[0] = d & 1 ? v[0] * c + far * s : v[0] * c - far * s;
    } else {
        #pragma unroll
        for (int i = 0; i < VEC; i += 2) {
            if (d + i >= dims) return;
            const float c = cs[d + i], s = cs[d + i + 1];
            const float a = v[i], b = v[i + 1];
            v[i] = a * c - b * s;
            v[i + 1] = b * c + a * s;
        }
    }
}

// columns c.. of row t plus their bias
template <int VEC, typename P>
DEV void biased(const Rows<P>& p, const float* bias, int64_t t, int c,
                float* v) {
    ldrow<VEC>(p, t, c, v);
    if (bias) {
        float b[VEC];
        ldv<VEC>(bias + c, b);
        #pragma unroll
        for (int i = 0; i < VEC; i++) v[i] += b[i];
    }
}

template <typename T, typename P, int VEC>
__global__ __launch_bounds__(256) void k_rope_qkv_append(
    T* __restrict__ q_out, T* __restrict__ kpool, T* __restrict__ vpool,
    Rows<P> p, const float* __restrict__ bias,
    const float* __restrict__ table, int dims,
    const int* __restrict__ slot, const int* __restrict__ pos,
    const int* __restrict__ ptab, int H, int G, int D, int V, int Dp, int Vp,
    int psz, int maxp)
{
    const int64_t t = blockIdx.x;
    const int nq = H * D, nk = G * D, n = nq + nk + G * V;
    const int ps = pos[t];
    const int64_t page = ptab[(int64_t)slot[t] * maxp + ps / psz];
    const int off = ps % psz;
    const float* cs = table + (int64_t)ps * dims;
    const int first = blockIdx.y * 256 + threadIdx.x;
    const int stride = gridDim.y * 256;
    for (int c = first * VEC; c < n; c += stride * VEC) {
        float v[VEC], far = 0.f;
        biased<VEC>(p, bias, t, c, v);
        if (c < nq + nk) {
            const int hc = c < nq ? c : c - nq;
            const int h = hc / D, d = hc % D;
            if (VEC == 1 && d < dims)
                biased<1>(p, bias, t, d & 1 ? c - 1 : c + 1, &far);
            turn<VEC>(v, far, d, dims, cs);
            if (c < nq) stv<VEC>(q_out + (t * H + h) * Dp + d, v);
            else stv<VEC>(kpool + ((page * G + h) * psz + off) * Dp + d, v);
        } else {
            const int hc = c - nq - nk;
            stv<VEC>(vpool + ((page * G + hc / V) * psz + off) * Vp + hc % V,
                     v);
        }
    }
    if (Dp > D)
        for (int i = first; i < H * (Dp - D); i += stride)
            stf(q_out + (t * H + i / (Dp - D)) * Dp + D + i % (Dp - D), 0.f);
}

extern "C" int rope_qkv_append(
    int f32, void* q_out, void* kpool, void* vpool, const void* p, int p32,
    int n_part, int64_t part_stride, int64_t ld, const void* bias,
    const void* table, int dims, const void* slot, const void* pos,
    const void* ptab, int T_rows, int H, int G, int D, int V, int Dp, int Vp,
    int psz, int maxp, hipStream_t stream)
{
    if (dims % 2 || dims > D || dims < 0) return (int)hipErrorInvalidValue;
    const int n = H * D + G * (D + V);
    const bool v4 = D % 4 == 0 && V % 4 == 0 && ld % 4 == 0
                    && part_stride % 4 == 0;
    const int per = 256 * (v4 ? 4 : 1);
    const int want = (n + per - 1) / per;
    const dim3 grid(T_rows, T_rows <= 256 ? want : (want + 3) / 4);
    #define RA(T, P, VE)                                                   \
        k_rope_qkv_append<T, P, VE><<<grid, 256, 0, stream>>>(             \
            (T*)q_out, (T*)kpool, (T*)vpool,                               \
            Rows<P>{(const P*)p, n_part, part_stride, ld},                 \
            (const float*)bias, (const float*)table, dims,                 \
            (const int*)slot, (const int*)pos, (const int*)ptab, H, G, D,  \
            V, Dp, Vp, psz, maxp)
    #define RA_V(T, P) do { if (v4) RA(T, P, 4); else RA(T, P, 1); } while (0)
    if (f32) RA_V(float, float);
    else if (p32) RA_V(bf16, float);
    else RA_V(bf16, bf16);
    #undef RA_V
    #undef RA
    return (int)hipGetLastError();
}

// A group of L lanes per head of a token: queries normed with qn and scaled by
// the head's gain, keys normed with kn, values normed without a weight; pairs
// (i, i + dims / 2) of queries and keys turn.  KEEP * L * VEC >= widths.
template <typename T, typename P, int VEC, int KEEP>
__global__ __launch_bounds__(256) void k_qkv_norm_rope(
    T* __restrict__ q_out, T* __restrict__ kpool, T* __restrict__ vpool,
    Rows<P> p, const float* __restrict__ qn, const float* __restrict__ kn,
    const float* __restrict__ gain, int vnorm, float eps,
    const float* __restrict__ table, int dims,
    const int* __restrict__ slot, const int* __restrict__ pos,
    const int* __restrict__ ptab, int H, int G, int D, int V, int Dp, int Vp,
    int psz, int maxp, int L)
{
    const int lane = threadIdx.x & (L - 1);
    const int64_t t = blockIdx.x;
    const int ps = pos[t], half = dims / 2;
    const int64_t page = ptab[(int64_t)slot[t] * maxp + ps / psz];
    const int off = ps % psz, step = gridDim.y * (256 / L);
    const float* cs = table + (int64_t)ps * dims;
    for (int unit = blockIdx.y * (256 / L) + threadIdx.x / L;
         unit < H + 2 * G; unit += step) {
        const bool is_q = unit < H, is_v = unit >= H + G;
        const int wide = is_v ? V : D;
        const int c0 = is_v ? (H + G) * D + (unit - H - G) * V : unit * D;
        const float* wt = is_v ? nullptr : is_q ? qn : kn;
        float x[KEEP][VEC], s = 0.f;
        #pragma unroll
        for (int j = 0; j < KEEP; j++) {
            const int c = (j * L + lane) * VEC;
            #pragma unroll
            for (int i = 0; i < VEC; i++) x[j][i] = 0.f;
            if (c < wide) ldrow<VEC>(p, t, c0 + c, x[j]);
            #pragma unroll
            for (int i = 0; i < VEC; i++) s += x[j][i] * x[j][i];
        }
        for (int o = L / 2; o; o >>= 1) s += __shfl_xor(s, o, 64);
        const float f = is_v && !vnorm ? 1.f : 1.f / sqrtf(s / wide + eps);
        const float up = is_q && gain ? gain[unit] : 1.f;
        T* dst = is_q ? q_out + (t * H + unit) * Dp
            : is_v ? vpool + ((page * G + unit - H - G) * psz + off) * Vp
                   : kpool + ((page * G + unit - H) * psz + off) * Dp;
        const int end = is_q ? Dp : wide;       // queries end in zeros
        #pragma unroll
        for (int j = 0; j < KEEP; j++) {
            const int c = (j * L + lane) * VEC;
            if (c >= end) continue;
            if (c < wide) {
                if (wt) {
                    float g[VEC];
                    ldv<VEC>(wt + c, g);
                    #pragma unroll
                    for (int i = 0; i < VEC; i++) x[j][i] *= g[i];
                }
                if (!is_v && c < dims) {
                    const bool low = c < half;
                    const int far = low ? c + half : c - half;
                    const int a = low ? c : far;
                    float y[VEC], g[VEC];
                    ldrow<VEC>(p, t, c0 + far, y);
                    ldv<VEC>(wt + far, g);
                    #pragma unroll
                    for (int i = 0; i < VEC; i++) {
                        const float co = cs[2 * (a + i)], si = cs[2 * (a + i) + 1];
                        x[j][i] = x[j][i] * co
                                  + (low ? -si : si) * y[i] * g[i];
                    }
                }
                #pragma unroll
                for (int i = 0; i < VEC; i++) x[j][i] *= f * up;
            }
            stv<VEC>(dst + c, x[j]);
        }
    }
}

extern "C" int qkv_norm_rope(
    int f32, void* q_out, void* kpool, void* vpool, const void* p, int p32,
    int n_part, int64_t part_stride, int64_t ld, const void* qn,
    const void* kn, const void* gain, int vnorm, float eps,
    const void* table, int dims, const void* slot, const void* pos,
    const void* ptab, int T_rows, int H, int G, int D, int V, int Dp, int Vp,
    int psz, int maxp, hipStream_t stream)
{
    if (dims % 2 || dims > D || dims < 0 || Dp > 256 || Vp > 256 || D > Dp
        || V > Vp)
        return (int)hipErrorInvalidValue;
    auto whole = [&](int n) {
        return D % n == 0 && V % n == 0 && dims % (2 * n) == 0 && ld % n == 0
               && part_stride % n == 0;
    };
    const int vec = whole(8) ? 8 : whole(4) ? 4 : 1;
    int L = 64;
    if (vec > 1)
        while (L > 4 && L / 2 * vec >= Dp && L / 2 * vec >= Vp) L /= 2;
    const int want = ((H + 2 * G) * L + 255) / 256;
    const dim3 grid(T_rows, T_rows <= 256 ? want : (want + 2) / 3);
    #define QN(T, P, VE, KE)                                               \
        k_qkv_norm_rope<T, P, VE, KE><<<grid, 256, 0, stream>>>(           \
            (T*)q_out, (T*)kpool, (T*)vpool,                               \
            Rows<P>{(const P*)p, n_part, part_stride, ld},                 \
            (const float*)qn, (const float*)kn, (const float*)gain, vnorm, \
            eps, (const float*)table, dims, (const int*)slot,              \
            (const int*)pos, (const int*)ptab, H, G, D, V, Dp, Vp, psz,    \
            maxp, L)
    #define QN_V(T, P)                                                     \
        do {                                                               \
            if (vec == 8) QN(T, P, 8, 1);                                  \
            else if (vec == 4) QN(T, P, 4, 1);                             \
            else QN(T, P, 1, 4);                                           \
        } while (0)
    if (f32) QN_V(float, float);
    else if (p32) QN_V(bf16, float);
    else QN_V(bf16, bf16);
    #undef QN_V
    #undef QN
    return (int)hipGetLastError();
}

// Projection columns: q [H, D + Dr] | latent [R] | shared key part [Dr].
// Block y == 0 of a token makes its cache row (RP wide), the others its
// queries.
template <typename T, typename P, int VEC>
__global__ __launch_bounds__(256) void k_latent_rope_append(
    T* __restrict__ q_out,              // [T, H, D + Dr]
    T* __restrict__ pool, Rows<P> p, const float* __restrict__ w,
    const float* __restrict__ table, const int* __restrict__ slot,
    const int* __restrict__ pos, const int* __restrict__ ptab, int H, int D,
    int Dr, int R, int RP, int psz, int maxp, float eps)
{
    const int64_t t = blockIdx.x;
    const int tid = threadIdx.x, DD = D + Dr, nq = H * DD;
    const int ps = pos[t];
    const float* cs = table + (int64_t)ps * Dr;
    if (blockIdx.y == 0) {
        __shared__ float red[4];
        const int64_t page = ptab[(int64_t)slot[t] * maxp + ps / psz];
        T* dst = pool + (page * psz + ps % psz) * RP;
        float v[VEC], s = 0.f;
        for (int c = tid * VEC; c < R; c += 256 * VEC) {
            ldrow<VEC>(p, t, nq + c, v);
            #pragma unroll
            for (int i = 0; i < VEC; i++) s += v[i] * v[i];
        }
        const float f = 1.f / sqrtf(block_sum<256>(s, red) / R + eps);
        const bool one = R <= 256 * VEC;
        for (int c = tid * VEC; c < R; c += 256 * VEC) {
            float a[VEC];
            if (!one) ldrow<VEC>(p, t, nq + c, v);
            ldv<VEC>(w + c, a);
            #pragma unroll
            for (int i = 0; i < VEC; i++) v[i] *= f * a[i];
            stv<VEC>(dst + c, v);
        }
        for (int c = tid * VEC; c < Dr; c += 256 * VEC) {
            float u[VEC], far = 0.f;
            ldrow<VEC>(p, t, nq + R + c, u);
            if (VEC == 1) ldrow<1>(p, t, nq + R + (c ^ 1), &far);
            turn<VEC>(u, far, c, Dr, cs);
            stv<VEC>(dst + R + c, u);
        }
        return;
    }
    const int first = (blockIdx.y - 1) * 256 + tid;
    const int stride = (gridDim.y - 1) * 256;
    for (int c = first * VEC; c < nq; c += stride * VEC) {
        const int d = c % DD - D;       // place in the rotated part
        float v[VEC], far = 0.f;
        ldrow<VEC>(p, t, c, v);
        if (d >= 0) {
            if (VEC == 1) ldrow<1>(p, t, d & 1 ? c - 1 : c + 1, &far);
            turn<VEC>(v, far, d, Dr, cs);
        }
        stv<VEC>(q_out + t * nq + c, v);
    }
}

extern "C" int latent_rope_append(
    int f32, void* q_out, void* pool, const void* p, int p32, int n_part,
    int64_t part_stride, int64_t ld, const void* w, const void* table,
    const void* slot, const void* pos, const void* ptab, int T_rows, int H,
    int D, int Dr, int R, int RP, int psz, int maxp, float eps,
    hipStream_t stream)
{
    if (Dr % 2 || R + Dr > RP) return (int)hipErrorInvalidValue;
    const bool v4 = D % 4 == 0 && Dr % 4 == 0 && R % 4 == 0 && RP % 4 == 0
                    && ld % 4 == 0 && part_stride % 4 == 0;
    const int per = 256 * (v4 ? 4 : 1);
    const int want = (H * (D + Dr) + per - 1) / per;
    const dim3 grid(T_rows, 1 + (T_rows <= 256 ? want : (want + 3) / 4));
    #define LR(T, P, VE)                                                   \
        k_latent_rope_append<T, P, VE><<<grid, 256, 0, stream>>>(          \
            (T*)q_out, (T*)pool,                                           \
            Rows<P>{(const P*)p, n_part, part_stride, ld},                 \
            (const float*)w, (const float*)table, (const int*)slot,        \
            (const int*)pos, (const int*)ptab, H, D, Dr, R, RP, psz, maxp, \
            eps)
    #define LR_V(T, P) do { if (v4) LR(T, P, 4); else LR(T, P, 1); } while (0)
    if (f32) LR_V(float, float);
    else if (p32) LR_V(bf16, float);
    else LR_V(bf16, bf16);
    #undef LR_V
    #undef LR
    return (int)hipGetLastError();
}
