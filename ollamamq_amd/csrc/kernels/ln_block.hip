// gfx950 row step between the products of blocks that norm after the sum:
//
//   x' = L(mult * x + scale * y; w, b)    residual stream, fp32
//   h  = L(x'; w2, b2), or x' itself      next operand
//
// L is the layer norm (mean and variance of the row).  x may be the residual
// stream or embedding rows; y one sublayer's result or the sum of two, each
// first divided by its root mean square and weighted; any of them may still
// be the partial sums of a split product.  One block per row, the row in
// registers, so mean and variance are two passes over registers.
#include "tile_mma.h"

// a result [T, W], or n_part partial sums of it part_stride apart
struct Src {
    const void* p;
    int f32, n_part;
    int64_t part_stride;
};
template <typename T, int VEC>
DEV void fold(const Src& s, int64_t row, int c, int W, float* v) {
    if (sizeof(T) == 4 || s.f32)
        ldrow<VEC>(Rows<float>{(const float*)s.p, s.n_part, s.part_stride, W},
                   row, c, v);
    else
        ldrow<VEC>(Rows<T>{(const T*)s.p, s.n_part, s.part_stride, W}, row, c,
                   v);
}

template <typename T, int BS, int NV, int VEC, bool FR>
__global__ __launch_bounds__(BS) void k_ln_residual(
    float* __restrict__ x_out,          // [n, W] or null
    T* __restrict__ h_out,              // [n, W], FR: fragment layout
    const float* __restrict__ x_in,     // [T, W], or null: embedding rows
    const T* __restrict__ embed, const int* __restrict__ tokens,
    Src ya, Src yb,                     // null: nothing to add
    const float* __restrict__ post_a,   // [W], or null: ya as it is, no yb
    const float* __restrict__ post_b, float share,
    const float* __restrict__ scale,    // [W] or null
    const float* __restrict__ w, const float* __restrict__ b, float mult,
    const float* __restrict__ w2, const float* __restrict__ b2,
    float eps, const int64_t* __restrict__ rows, int W)
{
    const int o = blockIdx.x, tid = threadIdx.x;
    const int64_t r = rows ? rows[o] : o;
    __shared__ float red[6][BS / 64];
    float x[NV][VEC];
    auto col = [&](int j) { return (j * BS + tid) * VEC; };
    auto squares = [&](const float (*v)[VEC]) {
        float s = 0.f;
        #pragma unroll
        for (int j = 0; j < NV; j++) {
            if (col(j) >= W) break;
            #pragma unroll
            for (int i = 0; i < VEC; i++) s += v[j][i] * v[j][i];
        }
        return s;
    };
    auto norm = [&](const float* gain, const float* bias, int at) {
        float s = 0.f;
        #pragma unroll
        for (int j = 0; j < NV; j++) {
            if (col(j) >= W) break;
            #pragma unroll
            for (int i = 0; i < VEC; i++) s += x[j][i];
        }
        const float mean = block_sum<BS>(s, red[at]) / W;
        #pragma unroll
        for (int j = 0; j < NV; j++)
            #pragma unroll
            for (int i = 0; i < VEC; i++) x[j][i] -= mean;
        const float f = 1.f / sqrtf(block_sum<BS>(squares(x), red[at + 1]) / W
                                    + eps);
        #pragma unroll
        for (int j = 0; j < NV; j++) {
            const int c = col(j);
            if (c >= W) break;
            float g[VEC], d[VEC];
            ldv<VEC>(gain + c, g);
            ldv<VEC>(bias + c, d);
            #pragma unroll
            for (int i = 0; i < VEC; i++) x[j][i] = x[j][i] * f * g[i] + d[i];
        }
    };
    #pragma unroll
    for (int j = 0; j < NV; j++) {
        const int c = col(j);
        if (c < W) {
            if (x_in) ldv<VEC>(x_in + r * W + c, x[j]);
            else ldv<VEC>(embed + (int64_t)tokens[r] * W + c, x[j]);
        } else
            #pragma unroll
            for (int i = 0; i < VEC; i++) x[j][i] = 0.f;
    }
    if (ya.p) {
        float u[NV][VEC], v[NV][VEC];
        #pragma unroll
        for (int j = 0; j < NV; j++) {
            const int c = col(j);
            if (c >= W) break;
            fold<T, VEC>(ya, r, c, W, u[j]);
            if (yb.p) fold<T, VEC>(yb, r, c, W, v[j]);
        }
        if (post_a) {
            const float fa = share / sqrtf(
                block_sum<BS>(squares(u), red[0]) / W + eps);
            const float fb = yb.p ? share / sqrtf(
                block_sum<BS>(squares(v), red[1]) / W + eps) : 0.f;
            #pragma unroll
            for (int j = 0; j < NV; j++) {
                const int c = col(j);
                if (c >= W) break;
                float p[VEC];
                ldv<VEC>(post_a + c, p);
                #pragma unroll
                for (int i = 0; i < VEC; i++) u[j][i] *= fa * p[i];
                if (yb.p) {
                    ldv<VEC>(post_b + c, p);
                    #pragma unroll
                    for (int i = 0; i < VEC; i++)
                        u[j][i] += v[j][i] * (fb * p[i]);
                }
            }
        }
        #pragma unroll
        for (int j = 0; j < NV; j++) {
            const int c = col(j);
            if (c >= W) break;
            float p[VEC];
            if (scale) ldv<VEC>(scale + c, p);
            else
                #pragma unroll
                for (int i = 0; i < VEC; i++) p[i] = 1.f;
            #pragma unroll
            for (int i = 0; i < VEC; i++)
                x[j][i] = mult * x[j][i] + p[i] * u[j][i];
        }
        norm(w, b, 2);
    }
    if (x_out)
        #pragma unroll
        for (int j = 0; j < NV; j++) {
            const int c = col(j);
            if (c < W) stv<VEC>(x_out + (int64_t)o * W + c, x[j]);
        }
    if (w2) norm(w2, b2, 4);
    #pragma unroll
    for (int j = 0; j < NV; j++) {
        const int c = col(j);
        if (c < W)
            stv<VEC>(h_out + (FR ? frag_row_off(o, c, W)
                                 : (int64_t)o * W + c), x[j]);
    }
}

extern "C" int ln_residual(
    int f32, void* x_out, void* h_out, const void* x_in, const void* embed,
    const void* tokens, const void* ya, int a32, int na, int64_t sa,
    const void* yb, int b32, int nb, int64_t sb, const void* post_a,
    const void* post_b, float share, const void* scale, const void* w,
    const void* b, float mult, const void* w2, const void* b2, float eps,
    const void* rows, int n, int W, int frag, hipStream_t stream)
{
    const bool v4 = W % 4 == 0;
    if ((ya && !(w && b)) || (yb && !(post_a && post_b))
        || (!x_in && !tokens) || (frag && (!v4 || f32)))
        return (int)hipErrorInvalidValue;
    const bool few = n <= 256;                  // a block a CU: shorter rows
    #define LN(T, BS, NV, V, F)                                            \
        k_ln_residual<T, BS, NV, V, F><<<n, BS, 0, stream>>>(              \
            (float*)x_out, (T*)h_out, (const float*)x_in, (const T*)embed, \
            (const int*)tokens, Src{ya, a32, na, sa}, Src{yb, b32, nb, sb},\
            (const float*)post_a, (const float*)post_b, share,             \
            (const float*)scale, (const float*)w, (const float*)b, mult,   \
            (const float*)w2, (const float*)b2, eps, (const int64_t*)rows, \
            W)
    #define LN_N(T, V, F)                                                  \
        do {                                                               \
            if (W <= 256 * V) LN(T, 256, 1, V, F);                         \
            else if (few && W <= 1024 * V) LN(T, 1024, 1, V, F);           \
            else if (W <= 512 * V) LN(T, 256, 2, V, F);                    \
            else if (W <= 1024 * V) LN(T, 256, 4, V, F);                   \
            else if (W <= 4096 * V) LN(T, 1024, 4, V, F);                  \
            else if (W <= 8192 * V) LN(T, 1024, 8, V, F);                  \
            else return (int)hipErrorInvalidValue;                         \
        } while (0)
    if (f32) { if (v4) LN_N(float, 4, false); else LN_N(float, 1, false); }
    else if (frag) LN_N(bf16, 4, true);
    else if (v4) LN_N(bf16, 4, false);
    else LN_N(bf16, 1, false);
    #undef LN_N
    #undef LN
    return (int)hipGetLastError();
}
