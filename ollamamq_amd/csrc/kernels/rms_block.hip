// gfx950 row steps between the products of RMS-normed blocks:
//
//   x' = x + mult * N(y) * post + shift   residual sum, fp32; without post
//                                         mult * y itself is added
//   h  = N(x') * pre, or x' itself        next operand
//
// N divides a row by its root mean square.  x may be the residual stream, the
// scaled embedding rows or nothing.  y may still be split: partial sums of a
// split-K product, or a token's expert outputs with their shares, are added
// up on the way in.  h may be followed by the token's embedding row, as the
// operand of a product over both.  One block per row, the row in registers.
// In decode the row kernel can also route: with the new row at hand it takes
// the few experts' logits and chooses.
//
// Also here: the split of a fused query/key/value projection with an RMS
// norm over all queries and over all keys of a token, and the append of keys
// and values to the paged pools; and the norm over all heads of a token, or
// of every head by itself, with a gate.
#include "route.h"

// sum_s share[s] * y[s * stride] (share null: all ones)
template <int VEC, typename P>
DEV void fold(const P* y, int n, int64_t stride, const float* share,
              float* v) {
    ldv<VEC>(y, v);
    if (share) {
        #pragma unroll
        for (int i = 0; i < VEC; i++) v[i] *= share[0];
    }
    for (int s = 1; s < n; s++) {
        float u[VEC];
        ldv<VEC>(y + s * stride, u);
        const float w = share ? share[s] : 1.f;
        #pragma unroll
        for (int i = 0; i < VEC; i++) v[i] += w * u[i];
    }
}

struct Route {
    const void* router;                 // [E, W], null: no routing
    int* chosen;                        // [n, top]
    float* share;
    int E, top;
};
#define ROUTE_MAX 16                    // experts

// RT: route, pre is null
template <typename T, typename P, int BS, int NV, int VEC, bool FR, bool RT>
__global__ __launch_bounds__(BS) void k_rms_residual(
    float* __restrict__ x_out,          // [n, W] or null
    T* __restrict__ h_out,              // [n, W], FR: fragment layout
    const float* __restrict__ x_in,     // [T, W], or null: embedding rows
    const T* __restrict__ embed, const int* __restrict__ tokens,
    float embed_scale,
    const P* __restrict__ y,            // null: nothing to add
    int n_part, int64_t part_stride, int64_t row_stride,
    const float* __restrict__ share,    // [T, n_part] or null
    const float* __restrict__ post, const float* __restrict__ pre,
    const float* __restrict__ shift, // [W] or null
    float mult, float eps, const int64_t* __restrict__ rows, int W,
    int tail,                           // h rows: [h, embedding row]
    int bare,                           // no x at all
    Route rt)
{
    const int o = blockIdx.x, tid = threadIdx.x;
    const int64_t r = rows ? rows[o] : o;
    __shared__ float red[2][BS / 64];
    float x[NV][VEC];
    auto col = [&](int j) { return (j * BS + tid) * VEC; };
    #pragma unroll
    for (int j = 0; j < NV; j++) {
        const int c = col(j);
        if (c >= W) break;
        if (x_in) ldv<VEC>(x_in + r * W + c, x[j]);
        else if (bare)
            #pragma unroll
            for (int i = 0; i < VEC; i++) x[j][i] = 0.f;
        else {
            ldv<VEC>(embed + (int64_t)tokens[r] * W + c, x[j]);
            #pragma unroll
            for (int i = 0; i < VEC; i++) x[j][i] *= embed_scale;
        }
    }
    if (y) {
        float v[NV][VEC], s = 0.f;
        #pragma unroll
        for (int j = 0; j < NV; j++) {
            const int c = col(j);
            if (c >= W) break;
            fold<VEC>(y + r * row_stride + c, n_part, part_stride,
                      share ? share + r * n_part : nullptr, v[j]);
            #pragma unroll
            for (int i = 0; i < VEC; i++) s += v[j][i] * v[j][i];
        }
        const float f = post
            ? mult / sqrtf(block_sum<BS>(s, red[0]) / W + eps) : mult;
        #pragma unroll
        for (int j = 0; j < NV; j++) {
            const int c = col(j);
            if (c >= W) break;
            float w[VEC];
            if (post) ldv<VEC>(post + c, w);
            else
                #pragma unroll
                for (int i = 0; i < VEC; i++) w[i] = 1.f;
            #pragma unroll
            for (int i = 0; i < VEC; i++) x[j][i] += f * v[j][i] * w[i];
        }
    }
    if (shift) {
        #pragma unroll
        for (int j = 0; j < NV; j++) {
            const int c = col(j);
            if (c >= W) break;
            float w[VEC];
            ldv<VEC>(shift + c, w);
            #pragma unroll
            for (int i = 0; i < VEC; i++) x[j][i] += w[i];
        }
    }
    const int HW = tail ? 2 * W : W;
    auto put = [&](int c, const float* v) {
        stv<VEC>(h_out + (FR ? frag_row_off(o, c, HW) : (int64_t)o * HW + c),
                 v);
    };
    float f = 1.f;
    if (pre) {
        float s = 0.f;
        #pragma unroll
        for (int j = 0; j < NV; j++) {
            if (col(j) >= W) break;
            #pragma unroll
            for (int i = 0; i < VEC; i++) s += x[j][i] * x[j][i];
        }
        f = 1.f / sqrtf(block_sum<BS>(s, red[1]) / W + eps);
    }
    #pragma unroll
    for (int j = 0; j < NV; j++) {
        const int c = col(j);
        if (c >= W) break;
        if (x_out) stv<VEC>(x_out + (int64_t)o * W + c, x[j]);
        if (pre) {
            float w[VEC];
            ldv<VEC>(pre + c, w);
            #pragma unroll
            for (int i = 0; i < VEC; i++) x[j][i] *= f * w[i];
        }
        put(c, x[j]);
        if (tail) {
            float e[VEC];
            ldv<VEC>(embed + (int64_t)tokens[r] * W + c, e);
            #pragma unroll
            for (int i = 0; i < VEC; i++) e[i] *= embed_scale;
            put(W + c, e);
        }
    }
    if constexpr (RT) {
        __shared__ float part[BS / 64][8], z[ROUTE_MAX];
        const T* router = reinterpret_cast<const T*>(rt.router);
        // logits of h, not of x: as the other router kernels see it
        #pragma unroll
        for (int j = 0; j < NV; j++)
            #pragma unroll
            for (int i = 0; i < VEC; i++)
                x[j][i] = col(j) < W ? (float)(T)x[j][i] : 0.f;
        for (int e0 = 0; e0 < rt.E; e0 += 8) {
            float s[8] = {};
            #pragma unroll
            for (int j = 0; j < NV; j++) {
                const int c = min(col(j), W - VEC);
                #pragma unroll
                for (int q = 0; q < 8; q++) {
                    float w[VEC];
                    ldv<VEC>(router + (int64_t)min(e0 + q, rt.E - 1) * W + c,
                             w);
                    #pragma unroll
                    for (int i = 0; i < VEC; i++) s[q] += x[j][i] * w[i];
                }
            }
            #pragma unroll
            for (int q = 0; q < 8; q++) {
                s[q] = wave_sum(s[q]);
                if ((tid & 63) == 0) part[tid >> 6][q] = s[q];
            }
            __syncthreads();
            if (tid < 8 && e0 + tid < rt.E) {
                float t = 0.f;
                #pragma unroll
                for (int i = 0; i < BS / 64; i++) t += part[i][tid];
                z[e0 + tid] = t;
            }
            __syncthreads();
        }
        if (tid < 16)
            choose(z, rt.E, rt.top, tid, rt.chosen + (int64_t)o * rt.top,
                   rt.share + (int64_t)o * rt.top, true);
    }
}

// y32: y is fp32 whatever the model's type is
extern "C" int rms_residual(
    int f32, void* x_out, void* h_out, const void* x_in, const void* embed,
    const void* tokens, float embed_scale, const void* y, int y32,
    int n_part, int64_t part_stride, int64_t row_stride, const void* share,
    const void* post, const void* pre, const void* shift, float mult,
    float eps, const void* rows, int n, int W, int tail, int bare, int frag,
    const void* router,
    void* chosen, void* route_share, int E, int top, hipStream_t stream)
{
    const bool v4 = W % 4 == 0;
    if ((bare && (x_in || !y)) || (tail && (!tokens || router)))
        return (int)hipErrorInvalidValue;
    if (frag && (!v4 || f32)) return (int)hipErrorInvalidValue;
    if (router && (!frag || pre || E > ROUTE_MAX || top > E))
        return (int)hipErrorInvalidValue;
    const bool few = n <= 256;                  // a block a CU: shorter rows
    const Route rt{router, (int*)chosen, (float*)route_share, E, top};
    #define RR(T, P, BS, NV, V, F)                                         \
        k_rms_residual<T, P, BS, NV, V, (F) != 0, (F) == 2>                \
            <<<n, BS, 0, stream>>>(                                        \
            (float*)x_out, (T*)h_out, (const float*)x_in, (const T*)embed, \
            (const int*)tokens, embed_scale, (const P*)y, n_part,          \
            part_stride, row_stride, (const float*)share,                  \
            (const float*)post, (const float*)pre, (const float*)shift,    \
            mult, eps, (const int64_t*)rows, W, tail, bare, rt)
    #define RR_N(T, P, V, F)                                               \
        do {                                                               \
            if (W <= 256 * V) RR(T, P, 256, 1, V, F);                      \
            else if (few && W <= 1024 * V) RR(T, P, 1024, 1, V, F);        \
            else if (W <= 512 * V) RR(T, P, 256, 2, V, F);                 \
            else if (W <= 1024 * V) RR(T, P, 256, 4, V, F);                \
            else if (W <= 4096 * V) RR(T, P, 1024, 4, V, F);               \
            else if (W <= 8192 * V) RR(T, P, 1024, 8, V, F);               \
            else return (int)hipErrorInvalidValue;                         \
        } while (0)
    #define RR_F(T, P)                                                     \
        do {                                                               \
            if (v4) RR_N(T, P, 4, 0);                                      \
            else RR_N(T, P, 1, 0);                                         \
        } while (0)
    if (f32) RR_F(float, float);
    else if (router && y32) RR_N(bf16, float, 4, 2);
    else if (router) RR_N(bf16, bf16, 4, 2);
    else if (frag && y32) RR_N(bf16, float, 4, 1);
    else if (frag) RR_N(bf16, bf16, 4, 1);
    else if (y32) RR_F(bf16, float);
    else RR_F(bf16, bf16);
    #undef RR_F
    #undef RR_N
    #undef RR
    return (int)hipGetLastError();
}

// ---------------------------------------------------------------------------
// One block per token.  p: q | k | v of that token (row_stride apart, n_part
// partial sums part_stride apart); q is normed into q_out [T, H, Dp], k into
// its page, v copied to its page.  NV > 0: the row stays in registers.
// ---------------------------------------------------------------------------
template <typename T, typename P, int BS, int NV, int VEC>
__global__ __launch_bounds__(BS) void k_qk_norm_append(
    T* __restrict__ q_out, T* __restrict__ kpool, T* __restrict__ vpool,
    const P* __restrict__ p, int n_part, int64_t part_stride,
    int64_t row_stride, const float* __restrict__ qn,
    const float* __restrict__ kn, const int* __restrict__ slot,
    const int* __restrict__ pos, const int* __restrict__ ptab,
    int H, int G, int D, int V, int Dp, int Vp, int psz, int maxp, float eps)
{
    const int64_t t = blockIdx.x;
    const int tid = threadIdx.x;
    const int nq = H * D, nk = G * D, n = nq + nk + G * V;
    const int ps = pos[t];
    const int64_t page = ptab[(int64_t)slot[t] * maxp + ps / psz];
    const int off = ps % psz;
    const P* row = p + t * row_stride;
    __shared__ float red[2][BS / 64];
    constexpr int KEEP = NV > 0 ? NV : 1;
    float v[KEEP][VEC];
    float sq = 0.f, sk = 0.f;
    auto count = [&](int c, const float* u) {
        float s = 0.f;
        #pragma unroll
        for (int i = 0; i < VEC; i++) s += u[i] * u[i];
        if (c < nq) sq += s;
        else if (c < nq + nk) sk += s;
    };
    if constexpr (NV > 0) {
        #pragma unroll
        for (int j = 0; j < NV; j++) {
            const int c = (j * BS + tid) * VEC;
            if (c >= n) break;
            fold<VEC>(row + c, n_part, part_stride, nullptr, v[j]);
            count(c, v[j]);
        }
    } else {
        for (int c = tid * VEC; c < nq + nk; c += BS * VEC) {
            fold<VEC>(row + c, n_part, part_stride, nullptr, v[0]);
            count(c, v[0]);
        }
    }
    const float fq = 1.f / sqrtf(block_sum<BS>(sq, red[0]) / nq + eps);
    const float fk = 1.f / sqrtf(block_sum<BS>(sk, red[1]) / nk + eps);
    auto put = [&](int c, float* u) {
        float w[VEC];
        if (c < nq) {
            ldv<VEC>(qn + c, w);
            #pragma unroll
            for (int i = 0; i < VEC; i++) u[i] *= fq * w[i];
            stv<VEC>(q_out + (t * H + c / D) * Dp + c % D, u);
        } else if (c < nq + nk) {
            c -= nq;
            ldv<VEC>(kn + c, w);
            #pragma unroll
            for (int i = 0; i < VEC; i++) u[i] *= fk * w[i];
            stv<VEC>(kpool + ((page * G + c / D) * psz + off) * Dp + c % D,
                     u);
        } else {
            c -= nq + nk;
            stv<VEC>(vpool + ((page * G + c / V) * psz + off) * Vp + c % V,
                     u);
        }
    };
    if constexpr (NV > 0) {
        #pragma unroll
        for (int j = 0; j < NV; j++) {
            const int c = (j * BS + tid) * VEC;
            if (c >= n) break;
            put(c, v[j]);
        }
    } else {
        for (int c = tid * VEC; c < n; c += BS * VEC) {
            fold<VEC>(row + c, n_part, part_stride, nullptr, v[0]);
            put(c, v[0]);
        }
    }
    if (Dp > D)
        for (int i = tid; i < H * (Dp - D); i += BS)
            stf(q_out + (t * H + i / (Dp - D)) * Dp + D + i % (Dp - D), 0.f);
}

extern "C" int qk_norm_append(
    int f32, void* q_out, void* kpool, void* vpool, const void* p, int p32,
    int n_part, int64_t part_stride, int64_t row_stride, const void* qn,
    const void* kn, const void* slot, const void* pos, const void* ptab,
    int T_rows, int H, int G, int D, int V, int Dp, int Vp, int psz,
    int maxp, float eps, hipStream_t stream)
{
    const int n = H * D + G * (D + V);
    const bool vec = D % 4 == 0 && V % 4 == 0 && row_stride % 4 == 0
                     && part_stride % 4 == 0;
    #define QK(T, P, BS, NV, VE)                                           \
        k_qk_norm_append<T, P, BS, NV, VE><<<T_rows, BS, 0, stream>>>(     \
            (T*)q_out, (T*)kpool, (T*)vpool, (const P*)p, n_part,          \
            part_stride, row_stride, (const float*)qn, (const float*)kn,   \
            (const int*)slot, (const int*)pos, (const int*)ptab, H, G, D,  \
            V, Dp, Vp, psz, maxp, eps)
    #define QK_N(T, P)                                                     \
        do {                                                               \
            if (!vec) QK(T, P, 256, 0, 1);                                 \
            else if (n > 8192) QK(T, P, 1024, 0, 4);                       \
            else if (T_rows > 512) QK(T, P, 256, 8, 4);                    \
            else QK(T, P, 1024, 2, 4);                                     \
        } while (0)
    if (f32) QK_N(float, float);
    else if (p32) QK_N(bf16, float);
    else QK_N(bf16, bf16);
    #undef QK_N
    #undef QK
    return (int)hipGetLastError();
}

// ---------------------------------------------------------------------------
// out = N(o) * w * sigmoid(gate), the norm over a token's whole row of N
// columns; o fp32, the gate a column range of a projection that may still be
// split.  One block per token.  NV > 0: the row stays in registers.
// ---------------------------------------------------------------------------
template <typename T, typename P, int BS, int NV, int VEC, bool FR>
__global__ __launch_bounds__(BS) void k_rms_gate(
    T* __restrict__ out, const float* __restrict__ o,
    const float* __restrict__ w, Rows<P> gate, int og, int N, float eps)
{
    const int64_t t = blockIdx.x;
    const int tid = threadIdx.x;
    const float* row = o + t * N;
    __shared__ float red[BS / 64];
    constexpr int KEEP = NV > 0 ? NV : 1;
    float v[KEEP][VEC], s = 0.f;
    auto count = [&](const float* u) {
        #pragma unroll
        for (int i = 0; i < VEC; i++) s += u[i] * u[i];
    };
    if constexpr (NV > 0) {
        #pragma unroll
        for (int j = 0; j < NV; j++) {
            const int c = (j * BS + tid) * VEC;
            if (c >= N) break;
            ldv<VEC>(row + c, v[j]);
            count(v[j]);
        }
    } else {
        for (int c = tid * VEC; c < N; c += BS * VEC) {
            ldv<VEC>(row + c, v[0]);
            count(v[0]);
        }
    }
    const float f = 1.f / sqrtf(block_sum<BS>(s, red) / N + eps);
    auto emit = [&](int c, float* u) {
        float a[VEC], g[VEC];
        ldv<VEC>(w + c, a);
        ldrow<VEC>(gate, t, og + c, g);
        #pragma unroll
        for (int i = 0; i < VEC; i++)
            u[i] *= f * a[i] * sigmoid_of<T>(g[i]);
        stv<VEC>(out + (FR ? frag_row_off(t, c, N) : t * N + c), u);
    };
    if constexpr (NV > 0) {
        #pragma unroll
        for (int j = 0; j < NV; j++) {
            const int c = (j * BS + tid) * VEC;
            if (c >= N) break;
            emit(c, v[j]);
        }
    } else {
        for (int c = tid * VEC; c < N; c += BS * VEC) {
            ldv<VEC>(row + c, v[0]);
            emit(c, v[0]);
        }
    }
}

extern "C" int rms_gate(
    int f32, void* out, const void* o, const void* w, const void* gate,
    int p32, int n_part, int64_t part_stride, int64_t ld, int og, int T_rows,
    int N, float eps, int frag, hipStream_t stream)
{
    const bool vec = N % 4 == 0 && og % 4 == 0 && ld % 4 == 0
                     && part_stride % 4 == 0;
    if (frag && (f32 || !vec || N % 64)) return (int)hipErrorInvalidValue;
    #define RG(T, P, BS, NV, VE, FR)                                       \
        k_rms_gate<T, P, BS, NV, VE, FR><<<T_rows, BS, 0, stream>>>(       \
            (T*)out, (const float*)o, (const float*)w,                     \
            Rows<P>{(const P*)gate, n_part, part_stride, ld}, og, N, eps)
    #define RG_N(T, P, FR)                                                 \
        do {                                                               \
            if (!vec) RG(T, P, 256, 0, 1, false);                          \
            else if (N <= 1024) RG(T, P, 256, 1, 4, FR);                   \
            else if (T_rows <= 256 && N <= 4096) RG(T, P, 1024, 1, 4, FR); \
            else if (N <= 2048) RG(T, P, 256, 2, 4, FR);                   \
            else if (N <= 4096) RG(T, P, 256, 4, 4, FR);                   \
            else if (N <= 8192) RG(T, P, 1024, 2, 4, FR);                  \
            else RG(T, P, 1024, 0, 4, FR);                                 \
        } while (0)
    if (f32) RG_N(float, float, false);
    else if (frag && p32) RG_N(bf16, float, true);
    else if (frag) RG_N(bf16, bf16, true);
    else if (p32) RG_N(bf16, float, false);
    else RG_N(bf16, bf16, false);
    #undef RG_N
    #undef RG
    return (int)hipGetLastError();
}

// ---------------------------------------------------------------------------
// out = N(mult * o) * w * gate, the norm over every head of V columns by
// itself; w is shared by the heads (w_stride 0), per head (V) or null; the
// gate the sigmoid or silu of a column range of a projection.  A group of L
// lanes per head of a token.
// ---------------------------------------------------------------------------
template <typename T, typename P, int VEC, bool FR>
__global__ __launch_bounds__(256) void k_head_gate(
    T* __restrict__ out, const float* __restrict__ o, float mult,
    const float* __restrict__ w, int w_stride, Rows<P> gate, int og,
    int silu, int H, int V, int L, float eps)
{
    const int lane = threadIdx.x & (L - 1);
    const int64_t t = blockIdx.x;
    const int per = 256 / L, step = gridDim.y * per;
    const bool one = V <= L * VEC;          // the head fits the lanes
    for (int h = blockIdx.y * per + threadIdx.x / L; h < H; h += step) {
        const float* row = o + (t * H + h) * V;
        float x[VEC], g[VEC], s = 0.f;
        for (int c = lane * VEC; c < V; c += L * VEC) {
            ldv<VEC>(row + c, x);
            if (one) ldrow<VEC>(gate, t, og + h * V + c, g);
            #pragma unroll
            for (int i = 0; i < VEC; i++) s += x[i] * x[i];
        }
        for (int k = L / 2; k; k >>= 1) s += __shfl_xor(s, k, 64);
        const float f = mult / sqrtf(s * (mult * mult / V) + eps);
        for (int c = lane * VEC; c < V; c += L * VEC) {
            if (!one) {
                ldv<VEC>(row + c, x);
                ldrow<VEC>(gate, t, og + h * V + c, g);
            }
            #pragma unroll
            for (int i = 0; i < VEC; i++)
                x[i] *= f * sigmoid_of<T>(g[i]) * (silu ? g[i] : 1.f);
            if (w) {
                ldv<VEC>(w + h * w_stride + c, g);
                #pragma unroll
                for (int i = 0; i < VEC; i++) x[i] *= g[i];
            }
            const int n = h * V + c;
            stv<VEC>(out + (FR ? frag_row_off(t, n, H * V)
                               : t * (int64_t)H * V + n), x);
        }
    }
}

extern "C" int head_gate(
    int f32, void* out, const void* o, float mult, const void* w,
    int w_stride, const void* gate, int p32, int n_part, int64_t part_stride,
    int64_t ld, int og, int silu, int T_rows, int H, int V, float eps,
    int frag, hipStream_t stream)
{
    const bool v4 = V % 4 == 0 && og % 4 == 0 && ld % 4 == 0
                    && part_stride % 4 == 0;
    if (frag && f32) return (int)hipErrorInvalidValue;
    int L = 64;
    while (L > 4 && L / 2 * (v4 ? 4 : 1) >= V) L /= 2;
    const int want = (H * L + 255) / 256;
    const dim3 grid(T_rows, T_rows <= 256 ? want : (want + 1) / 2);
    #define HG(T, P, VE, FR)                                               \
        k_head_gate<T, P, VE, FR><<<grid, 256, 0, stream>>>(               \
            (T*)out, (const float*)o, mult, (const float*)w, w_stride,     \
            Rows<P>{(const P*)gate, n_part, part_stride, ld}, og, silu,    \
            H, V, L, eps)
    #define HG_V(T, P, FR)                                                 \
        do { if (v4) HG(T, P, 4, FR); else HG(T, P, 1, FR); } while (0)
    if (f32) HG_V(float, float, false);
    else if (frag && p32) HG_V(bf16, float, true);
    else if (frag) HG_V(bf16, bf16, true);
    else if (p32) HG_V(bf16, float, false);
    else HG_V(bf16, bf16, false);
    #undef HG_V
    #undef HG
    return (int)hipGetLastError();
}
