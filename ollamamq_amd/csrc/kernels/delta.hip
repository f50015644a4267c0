// gfx950 delta rules: per head a [D, V] fp32 state that forgets per key
// channel, removes along one vector what another reads, and writes,
//
//   S_t = diag(g_t) S_(t-1) - e_t (z_t^T S_(t-1)) + k_t v_t^T,
//   o_t = S_t^T q_t.
//
// * the gated rule (GEN false), u the unit key and b the step size:
//     S <- diag(g) S,  S <- S + u (b (v - S^T u))^T
//   is z = g u and e = k = b u; queries, keys and values come through a short
//   causal convolution and silu, queries and keys are unit vectors;
// * the generalized rule (GEN true): z = u, e = a u and k the key itself.
//
// k_gated_rows / k_general_rows make what the recurrence reads and the
// projection does not hold: convolved rows, scales that make unit vectors,
// log decays and step sizes from low-rank projections, the gated rule's
// output gate.  Then
//
// * k_delta_step: a token at a time (decode, portions of a few tokens), the
//   state in registers;
// * k_delta_prep / k_delta_scan: chunks of 64 tokens.  With c_i the sum of
//   log decays up to token i of a chunk and w_i = z_i^T S_(i-1),
//     w + A_ze w = Z S_0 + A_zk V,         Z_i = z_i e^{c_i} / g_i,
//     o = Q S_0 + A_qk V - A_qe w,         Q_i = q_i e^{c_i},
//     S' = diag(e^{c_n}) S_0 + K^T V - E^T w,   K_j = k_j e^{c_n - c_j},
//   A_xy[i][j] = sum_d x_id y_jd e^{c_i - c_j} for j < i (j <= i for q, and
//   for z with c_(i-1)).  In the gated rule e = k, so only u = V - w enters.
//   prep makes the factors, the A and (I + A_ze)^-1 for all chunks at once;
//   scan walks a sequence's chunks with the state in registers, a block per
//   head and strip of value columns.  No exponent that meets data is
//   positive: sums are kept per 16-token part, a pair of parts is joined by
//   the decay between them.
//
// The results o [T, H, V] are fp32; the norm and gate that follow are
// k_head_gate.  A sequence starts where its position is 0: state and earlier
// inputs are then taken as zero and whatever the slot held is ignored.
#include "tile_mma.h"

template <typename T> DEV float softplus_of(float x) {
    const float e = exp_of<T>(-fabsf(x));
    if constexpr (sizeof(T) == 4) return fmaxf(x, 0.f) + log1pf(e);
    // log(1 + e), with a series where 1 + e would lose e
    const float s = e * (1.f + e * (-0.5f + e * (1.f / 3.f + e * -0.25f)));
    return fmaxf(x, 0.f) + (e < 0.03f ? s : __logf(1.f + e));
}
#define UNIT_EPS 1e-6f                // inside the root of a unit vector
#define LOG_ZERO (-104.f)             // e to this is zero in fp32
#define HALF_DECAY 0.6065306597126334f   // e^{-1/2}

// ---------------------------------------------------------------------------
// z = W u for 16 tokens and rows n0 .. n1 - 1 of W [N, rank], u (or its tanh)
// the projection's columns first.. of the lane's token t; rank and first are
// whole vectors of 8.  W is stored as operands, 16 rows by 32 columns after
// one another, rows filled up to 64 and columns to 32.  `emit` gets 16 rows
// at a time, four of them in a lane: z[i] is row n + i.  The operand is made
// once for all rows while rank <= 128.
// ---------------------------------------------------------------------------
template <typename T, typename P, bool TANH, typename E>
DEV void low_rank(const Rows<P>& p, int first, int rank,
                  const T* __restrict__ w, int n0, int n1, int64_t t,
                  E emit) {
    constexpr int NT = Terms<T>::N;
    const int lane = threadIdx.x & 63, g = lane >> 4;
    const int steps = (rank + 31) / 32;
    Frag<T> uf[4][NT];
    auto operand = [&](int r0) {
        float u[4][8] = {};
        for (int q = 0; q < p.n_part; q++) {
            const P* src = p.p + q * p.part_stride + t * p.ld + first;
            float x[4][8];
            #pragma unroll
            for (int s = 0; s < 4; s++)
                ldv<8>(src + min(r0 + s * 32 + g * 8, rank - 8), x[s]);
            #pragma unroll
            for (int s = 0; s < 4; s++)
                #pragma unroll
                for (int e = 0; e < 8; e++) u[s][e] += x[s][e];
        }
        #pragma unroll
        for (int s = 0; s < 4; s++)
            #pragma unroll
            for (int e = 0; e < 8; e++) {
                const bool in = r0 + s * 32 + g * 8 < rank;
                T y[NT];
                Terms<T>::split(in ? TANH ? tanh_of<T>(u[s][e]) : u[s][e]
                                   : 0.f, y);
                #pragma unroll
                for (int q = 0; q < NT; q++)
                    frag_set(uf[s][q], e, ldf(&y[q]));
            }
    };
    // in decode the weights are as far away as the operand: ask for them first
    constexpr bool EARLY = sizeof(P) > sizeof(T);
    Frag<T> wf[4][4];
    auto weights = [&](int n, int r0, int s) {
        #pragma unroll
        for (int j = 0; j < 4; j++)
            wf[s][j] = frag8(w + ((int64_t)((n / 16 + j) * steps
                                            + min(r0 / 32 + s, steps - 1))
                                  * 64 + lane) * 8);
    };
    if (!EARLY && rank <= 128) operand(0);
    for (int n = n0; n < n1; n += 64) {
        f32x4 z[4] = {};
        for (int r0 = 0; r0 < rank; r0 += 128) {
            if constexpr (EARLY) {
                #pragma unroll
                for (int s = 0; s < 4; s++) weights(n, r0, s);
            }
            if (rank > 128 || (EARLY && n == n0)) operand(r0);
            #pragma unroll
            for (int s = 0; s < 4; s++) {
                if constexpr (!EARLY) {
                    if (r0 + s * 32 >= rank) continue;
                    weights(n, r0, s);
                }
                #pragma unroll
                for (int j = 0; j < 4; j++)
                    #pragma unroll
                    for (int q = 0; q < NT; q++)
                        z[j] = mma(wf[s][j], uf[s][q], z[j]);
            }
        }
        #pragma unroll
        for (int j = 0; j < 4; j++) emit(n + j * 16 + g * 4, z[j]);
    }
}
// four results from column n on
template <typename T>
DEV void put4(T* out, int64_t t, int n, int N, const float* v) {
    if (N % 4 == 0) { if (n < N) stv<4>(out + t * N + n, v); }
    else
        #pragma unroll
        for (int i = 0; i < 4; i++)
            if (n + i < N) stf(out + t * N + n + i, v[i]);
}

// ---------------------------------------------------------------------------
// Waves of several roles, in this order: convolution of a strip of tokens of
// one sequence (a group of L lanes per head), decays and gates of 16 tokens
// and 64 channels, step sizes.
// ---------------------------------------------------------------------------
template <typename T, typename P> struct GatedRows {
    Rows<P> p;
    int T_rows, o_in, ob, oa, ra, og, rg;     // columns and ranks
    int H, G, D, V, C, taps;
    const float* conv;                // [taps, C], the current token's last
    float* cstate;                    // [slots, taps - 1, C]
    const int* slot; const int* pos;
    const int* strips;                // [n, 4] first row, rows, the portion's
                                      // first row and end; null: every row
    int n_strips;
    const T* a2; const float* rate; const float* dt; const T* g2;
    T* y;                             // [T, C]
    float* scales;                    // [T, 2G] of queries and keys
    float* decay;                     // [T, H*D], logarithms
    float* beta;                      // [T, H]
    T* gate;                          // [T, H*V]
    int L, n_conv, n_decay, n_gate;   // lanes per head; waves of a role
    int wide;                         // columns of a low-rank wave
};

template <typename T, typename P, int VEC, int KEEP, int TAPS>
DEV void conv_strip(const GatedRows<T, P>& a, int64_t item, int lane) {
    const int U = 2 * a.G + a.H, unit = (int)(item % U);
    const int s = (int)(item / U);
    if (s >= a.n_strips) return;
    int row = s, n = 1, p0 = s, p1 = s + 1;
    if (a.strips) {
        row = a.strips[s * 4], n = a.strips[s * 4 + 1];
        p0 = a.strips[s * 4 + 2], p1 = a.strips[s * 4 + 3];
    }
    const bool is_v = unit >= 2 * a.G;
    const int wide = is_v ? a.V : a.D;
    const int c0 = is_v ? 2 * a.G * a.D + (unit - 2 * a.G) * a.V
                        : unit * a.D;
    const int taps = TAPS ? TAPS : a.taps, C = a.C;
    const bool fresh = a.pos[p0] == 0;
    float* st = a.cstate + (int64_t)a.slot[p0] * (taps - 1) * C + c0;
    // the input of row r, which may lie before the portion
    auto input = [&](int r, int c, float* v) {
        if (r >= p0) ldrow<VEC>(a.p, r, a.o_in + c0 + c, v);
        else if (!fresh) ldv<VEC>(st + (int64_t)(taps - 1 + r - p0) * C + c,
                                  v);
        else
            #pragma unroll
            for (int i = 0; i < VEC; i++) v[i] = 0.f;
    };
    auto col = [&](int j) { return (j * a.L + lane) * VEC; };
    constexpr int TM = TAPS ? TAPS : 1;
    float x[TM][KEEP][VEC], wt[TM][KEEP][VEC];      // the last inputs
    if constexpr (TAPS > 0) {
        #pragma unroll
        for (int j = 0; j < KEEP; j++) {
            if (col(j) >= wide) break;
            #pragma unroll
            for (int m = 0; m < TAPS; m++)
                ldv<VEC>(a.conv + m * C + c0 + col(j), wt[m][j]);
            #pragma unroll
            for (int m = 1; m < TAPS; m++)
                input(row - TAPS + m, col(j), x[m][j]);
        }
    }
    // rows a few at a time, the next ones under way
    constexpr int NR = TAPS > 0 ? 4 : 1;
    float next[NR][KEEP][VEC], ahead[NR][KEEP][VEC];
    auto fetch = [&](int r0) {
        #pragma unroll
        for (int y = 0; y < NR; y++)
            #pragma unroll
            for (int j = 0; j < KEEP; j++)
                if (col(j) < wide)
                    ldrow<VEC>(a.p, min(r0 + y, row + n - 1),
                               a.o_in + c0 + col(j), next[y][j]);
    };
    if constexpr (TAPS > 0) fetch(row);
    for (int r0 = row; r0 < row + n; r0 += NR) {
        if constexpr (TAPS > 0) {
            #pragma unroll
            for (int y = 0; y < NR; y++)
                #pragma unroll
                for (int j = 0; j < KEEP; j++)
                    #pragma unroll
                    for (int i = 0; i < VEC; i++)
                        ahead[y][j][i] = next[y][j][i];
            if (r0 + NR < row + n) fetch(r0 + NR);
        }
        #pragma unroll
        for (int y = 0; y < NR; y++) {
            const int r = r0 + y;
            if (r >= row + n) break;
            float sq = 0.f;
            #pragma unroll
            for (int j = 0; j < KEEP; j++) {
                const int c = col(j);
                if (c >= wide) break;
                float v[VEC] = {};
                if constexpr (TAPS > 0) {
                    #pragma unroll
                    for (int m = 0; m + 1 < TAPS; m++)
                        #pragma unroll
                        for (int i = 0; i < VEC; i++)
                            x[m][j][i] = x[m + 1][j][i];
                    #pragma unroll
                    for (int i = 0; i < VEC; i++)
                        x[TAPS - 1][j][i] = ahead[y][j][i];
                    #pragma unroll
                    for (int m = 0; m < TAPS; m++)
                        #pragma unroll
                        for (int i = 0; i < VEC; i++)
                            v[i] += wt[m][j][i] * x[m][j][i];
                } else
                    for (int m = 0; m < taps; m++) {
                        float u[VEC], w[VEC];
                        input(r - taps + 1 + m, c, u);
                        ldv<VEC>(a.conv + m * C + c0 + c, w);
                        #pragma unroll
                        for (int i = 0; i < VEC; i++) v[i] += w[i] * u[i];
                    }
                #pragma unroll
                for (int i = 0; i < VEC; i++) {
                    v[i] = silu_of<T>(v[i]);
                    sq += v[i] * v[i];
                }
                stv<VEC>(a.y + (int64_t)r * C + c0 + c, v);
            }
            if (is_v) continue;
            for (int o = a.L / 2; o; o >>= 1) sq += __shfl_xor(sq, o, 64);
            if (lane == 0)
                a.scales[(int64_t)r * 2 * a.G + unit] =
                    (unit < a.G ? 1.f / sqrtf((float)a.D) : 1.f)
                    / sqrtf(sq + UNIT_EPS);
        }
    }
    // Every row that reads the state is in its portion's first strip, and
    // this lane alone reads and writes these channels of it.
    if (row != p0) return;
    for (int m = 0; m < taps - 1; m++)
        #pragma unroll
        for (int j = 0; j < KEEP; j++) {
            const int c = col(j);
            if (c >= wide) break;
            float v[VEC];
            input(p1 - taps + 1 + m, c, v);
            stv<VEC>(st + (int64_t)m * C + c, v);
        }
}

template <typename T, typename P, int VEC, int KEEP, int TAPS>
__global__ __launch_bounds__(256, sizeof(P) > sizeof(T) ? 2 : 4)
void k_gated_rows(GatedRows<T, P> a)
{
    const int lane = threadIdx.x & 63, lr = lane & 15, g = lane >> 4;
    int64_t w = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (w < a.n_conv) {
        conv_strip<T, P, VEC, KEEP, TAPS>(
            a, w * (64 / a.L) + lane / a.L, lane & (a.L - 1));
        return;
    }
    w -= a.n_conv;
    if (w < a.n_decay) {
        const int N = a.H * a.D, nc = (N + a.wide - 1) / a.wide;
        const int n0 = (int)(w % nc) * a.wide;
        const int64_t t = w / nc * 16 + lr;
        low_rank<T, P, false>(
            a.p, a.oa, a.ra, a.a2, n0, min(n0 + a.wide, N),
            min(t, (int64_t)a.T_rows - 1), [&](int n, f32x4 z) {
                if (t >= a.T_rows || n >= N) return;
                const bool whole = a.D % 4 == 0;    // four of one head
                float v[4], rate = a.rate[n / a.D];
                #pragma unroll
                for (int i = 0; i < 4; i++) {
                    const int m = min(n + i, N - 1);
                    if (!whole) rate = a.rate[m / a.D];
                    v[i] = fmaxf(LOG_ZERO,
                                 -rate * softplus_of<T>(z[i] + a.dt[m]));
                }
                put4(a.decay, t, n, N, v);
            });
        return;
    }
    w -= a.n_decay;
    if (w < a.n_gate) {
        const int N = a.H * a.V, nc = (N + a.wide - 1) / a.wide;
        const int n0 = (int)(w % nc) * a.wide;
        const int64_t t = w / nc * 16 + lr;
        low_rank<T, P, false>(
            a.p, a.og, a.rg, a.g2, n0, min(n0 + a.wide, N),
            min(t, (int64_t)a.T_rows - 1), [&](int n, f32x4 z) {
                if (t >= a.T_rows) return;
                const float v[4] = {z[0], z[1], z[2], z[3]};
                put4(a.gate, t, n, N, v);
            });
        return;
    }
    w -= a.n_gate;
    const int64_t i = w * 64 + lane;
    if (i >= (int64_t)a.T_rows * a.H) return;
    float x;
    ldrow<1>(a.p, i / a.H, a.ob + (int)(i % a.H), &x);
    a.beta[i] = sigmoid_of<T>(x);
}

// columns of a low-rank wave: many share the operand, few fill the chip
static int low_rank_cols(int T_rows) { return T_rows > 512 ? 256 : 64; }
static bool low_rank_ok(int first, int rank, int64_t ld, int64_t stride) {
    return rank >= 8 && rank % 8 == 0 && first % 8 == 0 && ld % 8 == 0
           && stride % 8 == 0;
}
static int low_rank_waves(int64_t tokens, int channels, int wide) {
    return (int)((tokens + 15) / 16 * ((channels + wide - 1) / wide));
}

// strips int32 [n, 4] (first row, rows, the portion's first row and end), a
// strip no shorter than taps - 1 unless its portion is; null: every row is a
// portion of its own.
extern "C" int gated_rows(
    int f32, const void* p, int p32, int n_part, int64_t part_stride,
    int64_t ld, int o_in, int ob, int oa, int ra, int og, int rg,
    const void* conv, int taps, void* cstate, const void* slot,
    const void* pos, const void* strips, int n_strips, const void* a2,
    const void* rate, const void* dt, const void* g2, void* y, void* scales,
    void* decay, void* beta, void* gate, int T_rows, int H, int G, int D,
    int V, hipStream_t stream)
{
    const int C = 2 * G * D + H * V, wide = D > V ? D : V;
    const bool v4 = D % 4 == 0 && V % 4 == 0 && o_in % 4 == 0 && ld % 4 == 0
                    && part_stride % 4 == 0;
    if (taps < 1 || !low_rank_ok(oa, ra, ld, part_stride)
        || !low_rank_ok(og, rg, ld, part_stride)
        || wide > (v4 ? 1024 : 256))
        return (int)hipErrorInvalidValue;
    const bool one = v4 && wide <= 256;     // a head fits 64 lanes at once
    int L = 64;
    if (one) while (L > 1 && L / 2 * 4 >= wide) L /= 2;
    const int64_t units = (int64_t)n_strips * (2 * G + H);
    const int n_conv = (int)((units * L + 63) / 64);
    const int cols = low_rank_cols(T_rows);
    const int n_decay = low_rank_waves(T_rows, H * D, cols);
    const int n_gate = low_rank_waves(T_rows, H * V, cols);
    const int64_t all = (int64_t)n_conv + n_decay + n_gate
                        + ((int64_t)T_rows * H + 63) / 64;
    const int grid = (int)((all + 3) / 4);
    #define GR(T, P, VE, KE, TA)                                           \
        k_gated_rows<T, P, VE, KE, TA><<<grid, 256, 0, stream>>>(          \
            GatedRows<T, P>{                                               \
                Rows<P>{(const P*)p, n_part, part_stride, ld}, T_rows,     \
                o_in, ob, oa, ra, og, rg, H, G, D, V, C, taps,             \
                (const float*)conv, (float*)cstate, (const int*)slot,      \
                (const int*)pos, (const int*)strips, n_strips,             \
                (const T*)a2, (const float*)rate, (const float*)dt,        \
                (const T*)g2, (T*)y, (float*)scales, (float*)decay,        \
                (float*)beta, (T*)gate, L, n_conv, n_decay, n_gate, cols})
    #define GR_V(T, P)                                                     \
        do {                                                               \
            if (one && taps == 4) GR(T, P, 4, 1, 4);                       \
            else if (one) GR(T, P, 4, 1, 0);                               \
            else if (v4) GR(T, P, 4, 4, 0);                                \
            else GR(T, P, 1, 4, 0);                                        \
        } while (0)
    if (f32) GR_V(float, float);
    else if (p32) GR_V(bf16, float);
    else GR_V(bf16, bf16);
    #undef GR_V
    #undef GR
    return (int)hipGetLastError();
}

#define KEY_ROWS 4
// Roles of the generalized rule: scales of unit keys (a group of L lanes per
// head), decays, and, for a projection in parts, its sum.
template <typename T, typename P> struct GeneralRows {
    Rows<P> p;
    int T_rows, ok, ow, rank, H, D;
    const T* w2; const float* w0;
    float* scales;                    // [T, H]
    float* decay;                     // [T, H*D], logarithms
    T* y;                             // [T, cols] or null
    int cols, L, n_key, n_decay;
    int wide;                         // columns of a low-rank wave
};

template <typename T, typename P, int VEC>
__global__ __launch_bounds__(256, sizeof(P) > sizeof(T) ? 2 : 3)
void k_general_rows(GeneralRows<T, P> a)
{
    const int lane = threadIdx.x & 63, lr = lane & 15, g = lane >> 4;
    int64_t w = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (w < a.n_key) {
        // one head of up to KEY_ROWS tokens, their loads side by side
        const int64_t u = w * (64 / a.L) + lane / a.L;
        const int64_t t0 = u / a.H * KEY_ROWS;
        if (t0 >= a.T_rows) return;
        const int l = lane & (a.L - 1), h = (int)(u % a.H);
        float s[KEY_ROWS] = {};
        for (int c = l * VEC; c < a.D; c += a.L * VEC) {
            float x[KEY_ROWS][VEC];
            #pragma unroll
            for (int y = 0; y < KEY_ROWS; y++)
                ldrow<VEC>(a.p, min(t0 + y, (int64_t)a.T_rows - 1),
                           a.ok + h * a.D + c, x[y]);
            #pragma unroll
            for (int y = 0; y < KEY_ROWS; y++)
                #pragma unroll
                for (int i = 0; i < VEC; i++) s[y] += x[y][i] * x[y][i];
        }
        #pragma unroll
        for (int y = 0; y < KEY_ROWS; y++) {
            for (int o = a.L / 2; o; o >>= 1)
                s[y] += __shfl_xor(s[y], o, 64);
            if (l == 0 && t0 + y < a.T_rows)
                a.scales[(t0 + y) * a.H + h] = 1.f / sqrtf(s[y] + UNIT_EPS);
        }
        return;
    }
    w -= a.n_key;
    if (w < a.n_decay) {
        const int N = a.H * a.D, nc = (N + a.wide - 1) / a.wide;
        const int n0 = (int)(w % nc) * a.wide;
        const int64_t t = w / nc * 16 + lr;
        low_rank<T, P, true>(
            a.p, a.ow, a.rank, a.w2, n0, min(n0 + a.wide, N),
            min(t, (int64_t)a.T_rows - 1), [&](int n, f32x4 z) {
                if (t >= a.T_rows) return;
                float v[4];
                #pragma unroll
                for (int i = 0; i < 4; i++)
                    v[i] = -HALF_DECAY
                           * sigmoid_of<T>(z[i] + a.w0[min(n + i, N - 1)]);
                put4(a.decay, t, n, N, v);
            });
        return;
    }
    if (!a.y) return;
    w -= a.n_decay;
    const int64_t i = (w * 64 + lane) * VEC;
    if (i >= (int64_t)a.T_rows * a.cols) return;
    float x[VEC];
    ldrow<VEC>(a.p, i / a.cols, (int)(i % a.cols), x);
    stv<VEC>(a.y + i, x);
}

extern "C" int general_rows(
    int f32, const void* p, int p32, int n_part, int64_t part_stride,
    int64_t ld, int ok, int ow, int rank, const void* w2, const void* w0,
    void* scales, void* decay, void* y, int cols, int T_rows, int H, int D,
    hipStream_t stream)
{
    const bool v4 = D % 4 == 0 && ok % 4 == 0 && ld % 4 == 0
                    && part_stride % 4 == 0 && cols % 4 == 0;
    if (!low_rank_ok(ow, rank, ld, part_stride))
        return (int)hipErrorInvalidValue;
    int L = 64;
    while (L > 1 && L / 2 * (v4 ? 4 : 1) >= D) L /= 2;
    const int64_t keys = (int64_t)((T_rows + KEY_ROWS - 1) / KEY_ROWS) * H;
    const int n_key = (int)((keys * L + 63) / 64);
    const int wide = low_rank_cols(T_rows);
    const int n_decay = low_rank_waves(T_rows, H * D, wide);
    const int64_t n_sum = y ? ((int64_t)T_rows * cols / (v4 ? 4 : 1) + 63)
                              / 64 : 0;
    const int grid = (int)((n_key + n_decay + n_sum + 3) / 4);
    #define GE(T, P, VE)                                                   \
        k_general_rows<T, P, VE><<<grid, 256, 0, stream>>>(                \
            GeneralRows<T, P>{                                             \
                Rows<P>{(const P*)p, n_part, part_stride, ld}, T_rows, ok, \
                ow, rank, H, D, (const T*)w2, (const float*)w0,            \
                (float*)scales, (float*)decay, (T*)y, cols, L, n_key,      \
                n_decay, wide})
    #define GE_V(T, P) do { if (v4) GE(T, P, 4); else GE(T, P, 1); } while (0)
    if (f32) GE_V(float, float);
    else if (p32) GE_V(bf16, float);
    else GE_V(bf16, bf16);
    #undef GE_V
    #undef GE
    return (int)hipGetLastError();
}

// ---------------------------------------------------------------------------
// What the recurrence reads.  Rows of x hold q, k [G, D], v [H, V] and, for
// the generalized rule, removal rates before their bias [H, D].
// ---------------------------------------------------------------------------
template <typename T> struct DeltaIn {
    const T* x;
    int64_t ld;
    int oq, ok, ov, oa;
    const float* qs;                  // scales of q [T, sld] or null
    const float* ks;                  // and of unit keys
    int sld;
    const float* decay;               // [T, H*D], logarithms
    const float* beta;                // [T, H], gated rule
    const float* a_bias;              // [H*D], generalized rule
    int H, G, D, V;
};

// What follows the recurrence: every head normed by itself, times the weight
// and the sigmoid of the gate.
template <typename T> struct HeadOut {
    const float* w;
    int w_stride;                     // 0: the heads share the weight
    const T* gate;
    int64_t ld;
    int og;
    float eps;
    int frag;
};

// One block per sequence, head and strip of VB value columns; a thread keeps
// NR rows of VEC columns of the state.  OUT: the strip is the whole head, its
// norm and gate are in the same kernel.
template <typename T, int VEC, int NR, bool GEN, bool OUT>
__global__ __launch_bounds__(256) void k_delta_step(
    void* __restrict__ out,             // [T, H, V] fp32; OUT: of type T
    DeltaIn<T> in, float* __restrict__ state,   // [slots, H, D, V]
    const int* __restrict__ slot, const int* __restrict__ pos,
    const int* __restrict__ spans,      // [n, 2] first row, rows; null: 1 row
    int VB, HeadOut<T> ho)
{
    const int H = in.H, D = in.D, V = in.V;
    const int h = blockIdx.y, hk = h / (H / in.G), tid = threadIdx.x;
    const int v0 = blockIdx.z * VB, nc = min(VB, V - v0);
    const int t0 = spans ? spans[blockIdx.x * 2] : blockIdx.x;
    const int nt = spans ? spans[blockIdx.x * 2 + 1] : 1;
    const int nv = nc / VEC;            // threads across a state row
    const int RG = 256 / nv;            // state rows side by side
    const int rg = tid / nv;
    const bool on = rg < RG;
    const int vt = tid % nv * VEC;
    extern __shared__ __attribute__((aligned(16))) float sm[];
    float* r_s = sm;                    // [RG][nc] what z reads
    float* o_s = r_s + 256 * VEC;       // [RG][nc] what q reads
    float* q_s = o_s + 256 * VEC;       // [D]
    float* k_s = q_s + D;
    float* z_s = k_s + D;
    float* e_s = z_s + D;
    float* g_s = e_s + D;
    float* S = state + ((int64_t)slot[t0] * H + h) * D * V + v0 + vt;
    float s[NR][VEC];
    const bool fresh = pos[t0] == 0;
    #pragma unroll
    for (int j = 0; j < NR; j++) {
        const int d = rg + j * RG;
        if (on && !fresh && d < D) ldv<VEC>(S + (int64_t)d * V, s[j]);
        else
            #pragma unroll
            for (int i = 0; i < VEC; i++) s[j][i] = 0.f;
    }
    for (int t = t0; t < t0 + nt; ++t) {
        const T* row = in.x + (int64_t)t * in.ld;
        const float qs = in.qs ? in.qs[(int64_t)t * in.sld + hk] : 1.f;
        const float ks = in.ks[(int64_t)t * in.sld + hk];
        const float beta = GEN ? 0.f : in.beta[(int64_t)t * H + h];
        // this thread's first gate, asked for early
        const T* gr = ho.gate + t * ho.ld + ho.og + h * V;
        float z = 0.f, hw = 0.f;
        if (OUT && tid < V) {
            z = ldf(gr + tid);
            hw = ho.w[h * ho.w_stride + tid];
        }
        for (int d = tid; d < D; d += 256) {
            const int c = h * D + d;
            const float k = ldf(row + in.ok + hk * D + d), u = k * ks;
            const float g = exp_of<T>(in.decay[(int64_t)t * H * D + c]);
            q_s[d] = ldf(row + in.oq + hk * D + d) * qs;
            g_s[d] = g;
            if (GEN) {
                const float a = sigmoid_of<T>(ldf(row + in.oa + c)
                                              + in.a_bias[c]);
                k_s[d] = k;
                z_s[d] = u;
                e_s[d] = a * u;
            } else {
                k_s[d] = e_s[d] = beta * u;
                z_s[d] = g * u;
            }
        }
        __syncthreads();
        float v[VEC], acc[VEC] = {};
        if (on) {
            ldv<VEC>(row + in.ov + h * V + v0 + vt, v);
            #pragma unroll
            for (int j = 0; j < NR; j++) {
                const int d = rg + j * RG;
                if (d >= D) break;
                #pragma unroll
                for (int i = 0; i < VEC; i++) acc[i] += z_s[d] * s[j][i];
            }
            stv<VEC>(r_s + rg * nc + vt, acc);
        }
        __syncthreads();
        if (on) {
            float r[VEC] = {}, f[VEC] = {};
            for (int y = 0; y < RG; y++) {
                float x[VEC];
                ldv<VEC>(r_s + y * nc + vt, x);
                #pragma unroll
                for (int i = 0; i < VEC; i++) r[i] += x[i];
            }
            #pragma unroll
            for (int j = 0; j < NR; j++) {
                const int d = rg + j * RG;
                if (d >= D) break;
                #pragma unroll
                for (int i = 0; i < VEC; i++) {
                    s[j][i] = g_s[d] * s[j][i] - e_s[d] * r[i]
                              + k_s[d] * v[i];
                    f[i] += q_s[d] * s[j][i];
                }
            }
            stv<VEC>(o_s + rg * nc + vt, f);
        }
        __syncthreads();
        float sq = 0.f;
        for (int c = tid; c < nc; c += 256) {
            float x = 0.f;
            for (int y = 0; y < RG; y++) x += o_s[y * nc + c];
            if (OUT) {
                o_s[c] = x;             // only this thread reads column c
                sq += x * x;
            } else ((float*)out)[((int64_t)t * H + h) * V + v0 + c] = x;
        }
        if constexpr (OUT) {
            __shared__ float red[4];
            const float f = 1.f / sqrtf(block_sum<256>(sq, red) / V + ho.eps);
            for (int c = tid; c < V; c += 256) {
                const int m = h * V + c;
                if (c != tid) {
                    z = ldf(gr + c);
                    hw = ho.w[h * ho.w_stride + c];
                }
                stf((T*)out + (ho.frag ? frag_row_off(t, m, H * V)
                                       : (int64_t)t * H * V + m),
                    o_s[c] * f * hw * sigmoid_of<T>(z));
            }
        }
    }
    #pragma unroll
    for (int j = 0; j < NR; j++) {
        const int d = rg + j * RG;
        if (on && d < D) stv<VEC>(S + (int64_t)d * V, s[j]);
    }
}

#define DELTA_IN(T)                                                        \
    DeltaIn<T>{(const T*)x, ld, oq, ok, ov, oa, (const float*)qs,          \
               (const float*)ks, sld, (const float*)decay,                 \
               (const float*)beta, (const float*)a_bias, H, G, D, V}

// threads across a strip of the state: the rest of the block covers the rows,
// 16 a thread
static int step_threads(int D) {
    int nv = 256;
    while (nv > 1 && 256 / nv * 16 < D) nv /= 2;
    return nv;
}
// value columns of a block, fewer while there are few blocks
static int step_strip(int n, int H, int D, int V, bool v4) {
    const int most = step_threads(D) * (v4 ? 4 : 1);
    int vb = most < V ? most : V;
    while (v4 && vb > 32 && vb % 8 == 0
           && (int64_t)n * H * ((V + vb - 1) / vb) < 512) vb /= 2;
    return vb;
}
// whether the step kernel takes whole heads and can norm and gate them
extern "C" int delta_whole(int n, int H, int D, int V, int ov, int64_t ld)
{
    return V % 4 == 0 && ov % 4 == 0 && ld % 4 == 0
           && step_strip(n, H, D, V, true) == V;
}

// whole: 0 leaves o [T, H, V] in fp32; 1 and 2 norm and gate it into o [T, H*V]
// of the model's type, 2 in fragment layout.
extern "C" int delta_step(
    int f32, int gen, void* o, const void* x, int64_t ld, int oq, int ok,
    int ov, int oa, const void* qs, const void* ks, int sld,
    const void* decay, const void* beta, const void* a_bias, void* state,
    const void* slot, const void* pos, const void* spans, int n, int H,
    int G, int D, int V, const void* norm, int norm_stride, const void* gate,
    int64_t gate_ld, int og, float eps, int whole, hipStream_t stream)
{
    const bool v4 = V % 4 == 0 && ov % 4 == 0 && ld % 4 == 0;
    const int vec = v4 ? 4 : 1;
    if (D < 1 || V < 1 || D > 2048) return (int)hipErrorInvalidValue;
    int vb = step_strip(n, H, D, V, v4);
    if (whole) {
        if (V > step_threads(D) * vec || (whole == 2 && f32))
            return (int)hipErrorInvalidValue;
        vb = V;
    }
    const int rows = 256 / (vb / vec), per = (D + rows - 1) / rows;
    const int lds = (2 * 256 * vec + 5 * D) * 4;
    dim3 grid(n, H, (V + vb - 1) / vb);
    #define DS_GO(T, VE, NR, GEN, OUT)                                     \
        k_delta_step<T, VE, NR, GEN, OUT><<<grid, 256, lds, stream>>>(     \
            o, DELTA_IN(T), (float*)state, (const int*)slot,               \
            (const int*)pos, (const int*)spans, vb,                        \
            HeadOut<T>{(const float*)norm, norm_stride, (const T*)gate,    \
                       gate_ld, og, eps, whole == 2})
    #define DS_O(T, VE, NR, GEN)                                           \
        do {                                                               \
            if (whole) DS_GO(T, VE, NR, GEN, true);                        \
            else DS_GO(T, VE, NR, GEN, false);                             \
        } while (0)
    #define DS_N(T, VE, GEN)                                               \
        do {                                                               \
            if (per <= 4) DS_O(T, VE, 4, GEN);                             \
            else DS_O(T, VE, 16, GEN);                                     \
        } while (0)
    #define DS_V(T, GEN)                                                   \
        do { if (v4) DS_N(T, 4, GEN); else DS_N(T, 1, GEN); } while (0)
    if (per > 16) return (int)hipErrorInvalidValue;
    if (f32) { if (gen) DS_V(float, true); else DS_V(float, false); }
    else { if (gen) DS_V(bf16, true); else DS_V(bf16, false); }
    #undef DS_V
    #undef DS_N
    #undef DS_O
    #undef DS_GO
    return (int)hipGetLastError();
}

// ---- chunks --------------------------------------------------------------
#define CH 64             // tokens of a chunk
#define SUB 16            // tokens of a part
#define XCDS 8
#define DB 32             // key channels of a prep pass
#define DS (DB + 4)       // LDS row strides
#define AS (CH + 4)
// largest sum of decay inside a part for which the part's own triangle may
// be factored (e^{c_i} e^{-c_j}, far inside the range of fp32); beyond it the
// pairs are taken one by one
#define SAFE 60.f

// An fp32 matrix as operand of products: in bf16 models two planes of bf16
// terms whose products leave out the smallest, else itself.
template <typename T> struct Wide;
template <> struct Wide<float> { f32x8s f; };
template <> struct Wide<bf16> { bf16x8 hi, lo; };
DEV Wide<float> ldw(const float* p, int64_t) { return {frag8(p)}; }
DEV Wide<bf16> ldw(const bf16* p, int64_t plane) {
    return {frag8(p), frag8(p + plane)};
}
DEV f32x4 mma(const Wide<float>& a, const Wide<float>& b, f32x4 c) {
    return mma(a.f, b.f, c);
}
DEV f32x4 mma(const Wide<bf16>& a, const Wide<bf16>& b, f32x4 c) {
    c = mma(a.lo, b.hi, c);
    c = mma(a.hi, b.lo, c);
    return mma(a.hi, b.hi, c);
}
// by a matrix of the model's type
DEV f32x4 mma(const Wide<float>& a, const f32x8s& b, f32x4 c) {
    return mma(a.f, b, c);
}
DEV f32x4 mma(const Wide<bf16>& a, bf16x8 b, f32x4 c) {
    return mma(a.hi, b, mma(a.lo, b, c));
}
// VEC consecutive values
template <typename T, int VEC>
DEV void stw(T* p, int64_t plane, const float* v) {
    float f[Terms<T>::N][VEC];
    #pragma unroll
    for (int i = 0; i < VEC; i++) {
        T t[Terms<T>::N];
        Terms<T>::split(v[i], t);
        #pragma unroll
        for (int q = 0; q < Terms<T>::N; q++) f[q][i] = ldf(&t[q]);
    }
    #pragma unroll
    for (int q = 0; q < Terms<T>::N; q++) stv<VEC>(p + q * plane, f[q]);
}
template <typename T> DEV void stw4(T* p, int64_t plane, f32x4 v) {
    const float f[4] = {v[0], v[1], v[2], v[3]};
    stw<T, 4>(p, plane, f);
}
// four values of the model's type, as they are in memory
template <typename T> struct Four;
template <> struct Four<float> { typedef f32x4 type; };
template <> struct Four<bf16> { typedef bf16x4 type; };

// Scratch per (chunk, head), each matrix of NT planes: Q [64][DP],
// Z [64][DP], K^T [DP][64], (E^T), inverse [64][64], A_qk, (A_zk, A_qe);
// then the fp32 decay of the whole chunk [DP].  Offsets in elements of T.
// A matrix is stored as the operands the scan reads, 16 rows by 32 columns
// after one another, so that a wave's loads are linear.
template <typename T, bool GEN, int DP> struct Unit {
    static constexpr int NT = Terms<T>::N;
    static constexpr int64_t TP = CH * DP, SP = CH * CH;    // planes
    static constexpr int64_t tall(int m) { return m * NT * TP; }
    static constexpr int64_t square(int m) {
        return tall(GEN ? 4 : 3) + m * NT * SP;
    }
    static constexpr int64_t fade = square(GEN ? 4 : 2);
    static constexpr int64_t floats = (GEN ? 4 : 3) * TP + (GEN ? 4 : 2) * SP
                                      + DP;
    DEV T* at(float* scr, int64_t i) { return (T*)(scr + i * floats); }
};
// element (r, c) of a matrix with `steps` operands to a row of them
DEV int oper_at(int r, int c, int steps) {
    return ((r / 16 * steps + c / 32) * 64 + c % 32 / 8 * 16 + r % 16) * 8
           + c % 8;
}
enum { TALL_Q, TALL_Z, TALL_K, TALL_E };
enum { SQ_INV, SQ_QK, SQ_ZK, SQ_QE };

// VEC: rows of x are whole vectors of 8 key channels
template <typename T, bool GEN, int DP, bool VEC>
__global__ __launch_bounds__(256) void k_delta_prep(
    float* __restrict__ scr, DeltaIn<T> in,
    const int* __restrict__ chunks)     // [n, 2] first row, rows
{
    typedef Unit<T, GEN, DP> Un;
    const int H = in.H, D = in.D;
    const int h = blockIdx.y, hk = h / (H / in.G), tid = threadIdx.x;
    const int lane = tid & 63, w = tid >> 6;
    const int lr = lane & 15, g = lane >> 4;
    const int t0 = chunks[blockIdx.x * 2], n = chunks[blockIdx.x * 2 + 1];
    T* un = Un::at(scr, (int64_t)blockIdx.x * H + h);
    float* fade = (float*)(un + Un::fade);
    constexpr int PL = CH * DS;
    extern __shared__ __attribute__((aligned(16))) float sm[];
    float* qe_s = sm;                   // [64][DS] q e^{c}, c from the part on
    float* ze_s = qe_s + PL;            // z e^{c} / g
    float* kt_s = ze_s + PL;            // k e^{part total - c}
    float* kn_s = kt_s + PL;            // k e^{-c}, or k
    float* x1_s = kn_s + PL;            // GEN: e e^{part total - c}; else q
    float* x2_s = x1_s + PL;            // GEN: e e^{-c}; else u
    float* c_s = x2_s + PL;             // gated rule: c
    float* et_s = GEN ? c_s : c_s + PL; // [4][DB] e^{part total}
    float* A_s = sm;                    // [64][AS] afterwards
    float* I_s = A_s + CH * AS;

    // a lane's token, and its eight channels of a pass
    const int tk = w * SUB + (lane >> 2), c8 = (lane & 3) * 8;
    const bool live = tk < n;
    const int64_t t = t0 + min(tk, n - 1);
    const T* qr = in.x + t * in.ld + in.oq + hk * D;
    const T* kr = in.x + t * in.ld + in.ok + hk * D;
    const T* ar = in.x + t * in.ld + in.oa + h * D;
    const float* cr = in.decay + (t * H + h) * D;
    const float on = live ? 1.f : 0.f;
    const float qs = on * (in.qs ? in.qs[t * in.sld + hk] : 1.f);
    const float ks = on * in.ks[t * in.sld + hk];
    const float beta = GEN ? 0.f : in.beta[t * H + h];
    Frag<T> qn, kn, an;                 // the next pass
    f32x8s cn;
    auto load = [&](int d) {
        if constexpr (VEC) {
            const int c = min(d, D - 8);
            qn = frag8(qr + c);
            kn = frag8(kr + c);
            if (GEN) an = frag8(ar + c);
            cn = frag8(cr + c);
        } else {
            qn = frag_guard(qr, d, D);
            kn = frag_guard(kr, d, D);
            if (GEN) an = frag_guard(ar, d, D);
            cn = frag_guard(cr, d, D);
        }
    };
    // of the six tiles below the diagonal (1,0) (2,1) (3,2) (2,0) (3,1)
    // (3,0) this wave makes numbers w and w + 4
    const int ti[6] = {1, 2, 3, 2, 3, 3}, tj[6] = {0, 1, 2, 0, 1, 0};
    // products of q and z with k (and e), a query on a lane: the wave's
    // diagonal tile, the tiles below the diagonal
    f32x4 dqk = {}, dzk = {}, dqe = {}, dze = {};
    f32x4 oqk[2] = {}, ozk[2] = {}, oqe[2] = {}, oze[2] = {};

    load(c8);
    for (int d0 = 0; d0 < DP; d0 += DB) {
        const int d = d0 + c8;
        float q[8], k[8], c[8], a[8];
        #pragma unroll
        for (int e = 0; e < 8; e++) {
            const float in_d = d + e < D ? 1.f : 0.f;
            q[e] = in_d * frag_get(qn, e);
            k[e] = in_d * frag_get(kn, e);
            c[e] = in_d * on * frag_get(cn, e);
            if (GEN)
                a[e] = sigmoid_of<T>(frag_get(an, e)
                                     + in.a_bias[h * D + min(d + e, D - 1)]);
        }
        if (d0 + DB < DP) load(d + DB);
        float own[8], tot[8];
        bool safe = true;
        #pragma unroll
        for (int e = 0; e < 8; e++) {
            own[e] = c[e];
            #pragma unroll
            for (int s = 4; s < 64; s *= 2) {       // tokens are 4 lanes apart
                const float y = __shfl_up(c[e], s, 64);
                if (lane >= s) c[e] += y;
            }
            tot[e] = __shfl(c[e], 60 + (lane & 3), 64);
            safe = safe && tot[e] > -SAFE;
        }
        safe = GEN || __all(safe);
        float qe[8], ze[8], kt[8], kn2[8], x1[8], x2[8];
        #pragma unroll
        for (int e = 0; e < 8; e++) {
            const float grow = exp_of<T>(c[e]);
            const float back = safe ? exp_of<T>(-c[e]) : 1.f;
            const float left = exp_of<T>(tot[e] - c[e]);
            const float u = k[e] * ks;
            const float kk = GEN ? k[e] * on : beta * u;
            qe[e] = q[e] * qs * grow;
            ze[e] = u * (GEN ? exp_of<T>(c[e] - own[e]) : grow);
            kt[e] = kk * left;
            kn2[e] = kk * back;
            x1[e] = GEN ? a[e] * u * left : q[e] * qs;
            x2[e] = GEN ? a[e] * u * back : u;
        }
        __syncthreads();                // the pass before is done with
        const int at = tk * DS + c8;
        stv<8>(qe_s + at, qe);
        stv<8>(ze_s + at, ze);
        stv<8>(kt_s + at, kt);
        stv<8>(kn_s + at, kn2);
        if (GEN || !safe) {
            stv<8>(x1_s + at, x1);
            stv<8>(x2_s + at, x2);
        }
        if (!GEN && !safe) stv<8>(c_s + at, c);
        if ((lane >> 2) == 0) {
            #pragma unroll
            for (int e = 0; e < 8; e++) tot[e] = exp_of<T>(tot[e]);
            stv<8>(et_s + w * DB + c8, tot);
        }
        __syncthreads();
        // factors that meet the state: the decay of the parts before joins
        // q and z, that of the parts after k and e
        {
            float before[8];
            #pragma unroll
            for (int e = 0; e < 8; e++) before[e] = 1.f;
            for (int s = 0; s < w; s++) {
                float f[8];
                ldv<8>(et_s + s * DB + c8, f);
                #pragma unroll
                for (int e = 0; e < 8; e++) before[e] *= f[e];
            }
            #pragma unroll
            for (int e = 0; e < 8; e++) {
                qe[e] *= before[e];
                ze[e] *= before[e];
            }
            stw<T, 8>(un + Un::tall(TALL_Q) + oper_at(tk, d, DP / 32), Un::TP,
                      qe);
            stw<T, 8>(un + Un::tall(TALL_Z) + oper_at(tk, d, DP / 32), Un::TP,
                      ze);
            // transposed: eight tokens of a channel
            const int tt = (tid & 7) * 8, ch = tid >> 3;
            float after = 1.f, y[8];
            for (int s = tt / SUB + 1; s < 4; s++) after *= et_s[s * DB + ch];
            #pragma unroll
            for (int i = 0; i < 8; i++)
                y[i] = after * kt_s[(tt + i) * DS + ch];
            stw<T, 8>(un + Un::tall(TALL_K) + oper_at(d0 + ch, tt, 2), Un::TP,
                      y);
            if (GEN) {
                #pragma unroll
                for (int i = 0; i < 8; i++)
                    y[i] = after * x1_s[(tt + i) * DS + ch];
                stw<T, 8>(un + Un::tall(TALL_E) + oper_at(d0 + ch, tt, 2),
                          Un::TP, y);
            }
            if (tid < DB)
                fade[d0 + tid] = et_s[tid] * et_s[DB + tid]
                                 * et_s[2 * DB + tid] * et_s[3 * DB + tid];
        }
        // tiles below the diagonal
        #pragma unroll
        for (int x = 0; x < 2; x++) {
            const int id = w + x * 4;
            if (id >= 6) continue;
            const int I = ti[id], J = tj[id];
            f32x8s qa = frag8(qe_s + (I * SUB + lr) * DS + g * 8);
            f32x8s za = frag8(ze_s + (I * SUB + lr) * DS + g * 8);
            for (int s = J + 1; s < I; s++) {
                const f32x8s f = frag8(et_s + s * DB + g * 8);
                qa.lo *= f.lo; qa.hi *= f.hi;
                za.lo *= f.lo; za.hi *= f.hi;
            }
            const f32x8s kb = frag8(kt_s + (J * SUB + lr) * DS + g * 8);
            oqk[x] = mma(kb, qa, oqk[x]);
            ozk[x] = mma(kb, za, ozk[x]);
            if (GEN) {
                const f32x8s eb = frag8(x1_s + (J * SUB + lr) * DS + g * 8);
                oqe[x] = mma(eb, qa, oqe[x]);
                oze[x] = mma(eb, za, oze[x]);
            }
        }
        // the part's own triangle
        if (safe) {
            const int r = (w * SUB + lr) * DS + g * 8;
            const f32x8s qa = frag8(qe_s + r), za = frag8(ze_s + r);
            const f32x8s kb = frag8(kn_s + r);
            dqk = mma(kb, qa, dqk);
            dzk = mma(kb, za, dzk);
            if (GEN) {
                const f32x8s eb = frag8(x2_s + r);
                dqe = mma(eb, qa, dqe);
                dze = mma(eb, za, dze);
            }
        } else {
            // lane: column lr (the query), rows 4g + i (the key)
            for (int e = 0; e < DB; e++) {
                const int oi = (w * SUB + lr) * DS + e;
                const float ci = c_s[oi], qi = x1_s[oi], zi = x2_s[oi];
                #pragma unroll
                for (int i = 0; i < 4; i++) {
                    const int oj = (w * SUB + g * 4 + i) * DS + e;
                    const float f = kn_s[oj]
                                    * exp_of<T>(fminf(ci - c_s[oj], 0.f));
                    dqk[i] += qi * f;
                    dzk[i] += zi * f;
                }
            }
        }
    }
    // A_ze to LDS, the others to memory; the gated rule's A_ze is A_zk
    __syncthreads();
    auto place = [&](int m, int I, int J, f32x4 v) {
        stw4(un + Un::square(m) + oper_at(I * SUB + lr, J * SUB + g * 4, 2),
             Un::SP, v);
    };
    auto keep = [&](int I, int J, f32x4 v) {
        *reinterpret_cast<f32x4*>(
            A_s + (I * SUB + lr) * AS + J * SUB + g * 4) = v;
    };
    #pragma unroll
    for (int i = 0; i < 4; i++) {
        if (g * 4 + i > lr) dqk[i] = dqe[i] = 0.f;
        if (g * 4 + i >= lr) dzk[i] = dze[i] = 0.f;
    }
    place(SQ_QK, w, w, dqk);
    keep(w, w, GEN ? dze : dzk);
    if (GEN) {
        place(SQ_ZK, w, w, dzk);
        place(SQ_QE, w, w, dqe);
    }
    for (int J = w + 1; J < 4; J++) {
        const f32x4 none = {};
        place(SQ_QK, w, J, none);
        if (GEN) {
            place(SQ_ZK, w, J, none);
            place(SQ_QE, w, J, none);
        }
    }
    #pragma unroll
    for (int x = 0; x < 2; x++) {
        const int id = w + x * 4;
        if (id >= 6) continue;
        place(SQ_QK, ti[id], tj[id], oqk[x]);
        keep(ti[id], tj[id], GEN ? oze[x] : ozk[x]);
        if (GEN) {
            place(SQ_ZK, ti[id], tj[id], ozk[x]);
            place(SQ_QE, ti[id], tj[id], oqe[x]);
        }
    }
    __syncthreads();
    // (I + A)^-1: a column a lane inside the diagonal blocks, then block by
    // block below them
    {
        const float* A = A_s + w * SUB * AS + w * SUB;
        float x[SUB];
        #pragma unroll
        for (int i = 0; i < SUB; i++) {
            float y = i == lr ? 1.f : 0.f;
            #pragma unroll
            for (int j = 0; j < i; j++) y -= A[i * AS + j] * x[j];
            x[i] = y;
        }
        #pragma unroll
        for (int i = 0; i < SUB; i++)
            if (i / 4 == g) I_s[(w * SUB + i) * AS + w * SUB + lr] = x[i];
    }
    __syncthreads();
    auto below = [&](int I, int J) {
        f32x4 y = {}, z = {};
        for (int K = J; K < I; K++) {
            const f32x4 a = *reinterpret_cast<const f32x4*>(
                A_s + (I * SUB + lr) * AS + K * SUB + g * 4);
            #pragma unroll
            for (int e = 0; e < 4; e++)
                y = __builtin_amdgcn_mfma_f32_16x16x4f32(
                    a[e], I_s[(K * SUB + g * 4 + e) * AS + J * SUB + lr], y,
                    0, 0, 0);
        }
        const f32x4 a = *reinterpret_cast<const f32x4*>(
            I_s + (I * SUB + lr) * AS + I * SUB + g * 4);
        #pragma unroll
        for (int e = 0; e < 4; e++)
            z = __builtin_amdgcn_mfma_f32_16x16x4f32(a[e], y[e], z, 0, 0, 0);
        #pragma unroll
        for (int i = 0; i < 4; i++)
            I_s[(I * SUB + g * 4 + i) * AS + J * SUB + lr] = -z[i];
    };
    #pragma unroll
    for (int s = 1; s < 4; s++) {
        if (w + s < 4) below(w + s, w);
        __syncthreads();
    }
    for (int i = tid; i < CH * CH / 8; i += 256) {
        const int r = i / (CH / 8), c = i % (CH / 8) * 8;
        float v[8] = {};
        if (c / SUB <= r / SUB) ldv<8>(I_s + r * AS + c, v);
        stw<T, 8>(un + Un::square(SQ_INV) + oper_at(r, c, 2), Un::SP, v);
    }
}

// memory accesses stay on their side
DEV void keep_order() { asm volatile("" ::: "memory"); }

// A sequence's chunks in order, one block per 16*VC value columns, the state
// in registers (NS: 16-row tiles a wave, D <= 64 * NS); wave w has tokens
// 16 w .. of a chunk.  What several waves need goes through LDS, transposed:
// the state, v, what w is solved from and w itself.  The strips of a head are
// neighbours on one XCD, whose L2 they share the factors through.  VEC: rows
// of x are whole vectors of 4 value columns.
template <typename T, int NS, int VC, bool GEN, bool VEC>
__global__ __launch_bounds__(256) void k_delta_scan(
    float* __restrict__ o,              // [T, H, V]
    float* __restrict__ scr, DeltaIn<T> in, float* __restrict__ state,
    const int* __restrict__ slot, const int* __restrict__ pos,
    const int* __restrict__ chunks,     // [n, 2]
    const int* __restrict__ seqs,       // [m, 2] first chunk, chunks
    int n_seqs)
{
    constexpr int DP = NS * 64;
    typedef Unit<T, GEN, DP> Un;
    typedef typename Four<T>::type Raw;
    constexpr int W = VC * 16, NT = Terms<T>::N, PAD = 16 / sizeof(T);
    constexpr int KS = DP + PAD, TS = CH + PAD;
    constexpr int NQ = NS * 2;          // 32-channel steps over D
    constexpr int SP = W * KS, VP = W * TS;         // planes
    const int H = in.H, D = in.D, V = in.V, tid = threadIdx.x;
    const int strips = (V + W - 1) / W, place = blockIdx.x / XCDS;
    const int head = place / strips * XCDS + blockIdx.x % XCDS;
    if (head >= n_seqs * H) return;
    const int seq = head / H, h = head % H, v0 = place % strips * W;
    const int lane = tid & 63;
    const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int lr = lane & 15, g = lane >> 4;
    const int c0 = seqs[seq * 2], nc = seqs[seq * 2 + 1];
    const int first = chunks[c0 * 2];
    float* St = state + ((int64_t)slot[first] * H + h) * D * V;
    extern __shared__ __attribute__((aligned(16))) char smem[];
    T* S_s = reinterpret_cast<T*>(smem);      // [NT][W][KS] state
    T* r_s = S_s + NT * SP;                   // [NT][W][TS] right-hand side
    T* u_s = r_s + NT * VP;                   // [NT][W][TS] solution
    T* v_s = u_s + NT * VP;                   // [GEN ? 2 : 1][W][TS]

    f32x4 S[NS][VC];
    const bool fresh = pos[first] == 0;
    #pragma unroll
    for (int x = 0; x < NS; x++)
        #pragma unroll
        for (int c = 0; c < VC; c++)
            #pragma unroll
            for (int i = 0; i < 4; i++) {
                const int d = (w + x * 4) * 16 + g * 4 + i;
                const int v = v0 + c * 16 + lr;
                S[x][c][i] = (fresh || d >= D || v >= V)
                                 ? 0.f : St[(int64_t)d * V + v];
            }

    // operands in flight, loaded as soon as those before are used
    Wide<T> zf[NQ], qf[NQ], inv[2], aqk[2], azk[2], aqe[2];
    Wide<T> kf[NS][2], ef[NS][2];
    f32x4 e4[NS];
    Raw vv[VC];
    auto unit = [&](int ci) { return Un::at(scr, (int64_t)ci * H + h); };
    auto load_zq = [&](int ci) {
        const T* u = unit(ci) + w * NQ * 512 + lane * 8;
        #pragma unroll
        for (int d = 0; d < NQ; d++) {
            zf[d] = ldw(u + Un::tall(TALL_Z) + d * 512, Un::TP);
            qf[d] = ldw(u + Un::tall(TALL_Q) + d * 512, Un::TP);
        }
    };
    auto load_square = [&](int ci, int m, Wide<T>* f) {
        const T* u = unit(ci) + Un::square(m) + w * 1024 + lane * 8;
        #pragma unroll
        for (int j = 0; j < 2; j++) f[j] = ldw(u + j * 512, Un::SP);
    };
    auto load_fade = [&](int ci) {
        const float* fd = (const float*)(unit(ci) + Un::fade) + w * 16
                          + g * 4;
        #pragma unroll
        for (int x = 0; x < NS; x++)
            e4[x] = *reinterpret_cast<const f32x4*>(fd + x * 64);
    };
    auto load_k = [&](int ci) {
        const T* u = unit(ci) + w * 1024 + lane * 8;
        #pragma unroll
        for (int x = 0; x < NS; x++) {
            #pragma unroll
            for (int j = 0; j < 2; j++) {
                const int at = (x * 8 + j) * 512;
                kf[x][j] = ldw(u + Un::tall(TALL_K) + at, Un::TP);
                if (GEN) ef[x][j] = ldw(u + Un::tall(TALL_E) + at, Un::TP);
            }
        }
    };
    // token `lane` of a chunk, columns (wave * VC + q) * 4
    auto load_v = [&](int ci) {
        const int t0 = chunks[ci * 2], n = chunks[ci * 2 + 1];
        const T* r = in.x + (int64_t)(t0 + min(lane, n - 1)) * in.ld + in.ov
                     + h * V;
        #pragma unroll
        for (int q = 0; q < VC; q++) {
            const int c = v0 + (w * VC + q) * 4;
            if constexpr (VEC)
                vv[q] = *reinterpret_cast<const Raw*>(r + min(c, V - 4));
            else
                #pragma unroll
                for (int e = 0; e < 4; e++)
                    vv[q][e] = ldf(r + min(c + e, V - 1));
        }
    };
    auto wide_at = [&](const T* s, int c, int j) {
        return ldw(s + (c * 16 + lr) * TS + j * 32 + g * 8, VP);
    };
    // in the order of the loop, so that its waits fit the first chunk too
    load_v(c0);
    load_fade(c0);
    keep_order();
    load_zq(c0);
    keep_order();
    if (GEN) {
        load_square(c0, SQ_ZK, azk);
        load_square(c0, SQ_QK, aqk);
        keep_order();
    }
    load_square(c0, SQ_INV, inv);
    keep_order();
    load_square(c0, GEN ? SQ_QE : SQ_QK, GEN ? aqe : aqk);
    keep_order();
    load_k(c0);
    keep_order();

    for (int ci = c0; ci < c0 + nc; ++ci) {
        const int t0 = chunks[ci * 2], n = chunks[ci * 2 + 1];
        const int nx = min(ci + 1, c0 + nc - 1);
        T* vb = GEN && (ci & 1) ? v_s + VP : v_s;
        #pragma unroll
        for (int q = 0; q < VC; q++)
            #pragma unroll
            for (int e = 0; e < 4; e++) {
                const int c = (w * VC + q) * 4 + e;
                stf(vb + c * TS + lane, lane < n && v0 + c < V
                                            ? (float)vv[q][e] : 0.f);
            }
        #pragma unroll
        for (int x = 0; x < NS; x++) {
            const int d = (w + x * 4) * 16 + g * 4;
            #pragma unroll
            for (int c = 0; c < VC; c++)
                stw4(S_s + (c * 16 + lr) * KS + d, SP, S[x][c]);
        }
        #pragma unroll
        for (int x = 0; x < NS; x++)
            #pragma unroll
            for (int c = 0; c < VC; c++) S[x][c] *= e4[x];
        lds_barrier();
        load_v(nx);
        load_fade(nx);
        keep_order();
        // what z and q read from the state before the chunk
        f32x4 az[VC] = {}, ao[VC] = {};
        #pragma unroll
        for (int d = 0; d < NQ; d++)
            #pragma unroll
            for (int c = 0; c < VC; c++) {
                const Wide<T> b = ldw(S_s + (c * 16 + lr) * KS + d * 32
                                      + g * 8, SP);
                az[c] = mma(zf[d], b, az[c]);
                ao[c] = mma(qf[d], b, ao[c]);
            }
        load_zq(nx);
        if (GEN) {
            #pragma unroll
            for (int j = 0; j < 2; j++)
                #pragma unroll
                for (int c = 0; c < VC; c++) {
                    const Frag<T> b = frag8(vb + (c * 16 + lr) * TS + j * 32
                                            + g * 8);
                    az[c] = mma(azk[j], b, az[c]);
                    ao[c] = mma(aqk[j], b, ao[c]);
                }
            load_square(nx, SQ_ZK, azk);
            load_square(nx, SQ_QK, aqk);
        }
        #pragma unroll
        for (int c = 0; c < VC; c++) {
            const int at = (c * 16 + lr) * TS + w * 16 + g * 4;
            if (!GEN) {
                float f[4];
                ldv<4>(vb + at, f);
                #pragma unroll
                for (int i = 0; i < 4; i++) az[c][i] = f[i] - az[c][i];
            }
            stw4(r_s + at, VP, az[c]);
        }
        lds_barrier();
        f32x4 u[VC] = {};
        #pragma unroll
        for (int j = 0; j < 2; j++)
            #pragma unroll
            for (int c = 0; c < VC; c++)
                u[c] = mma(inv[j], wide_at(r_s, c, j), u[c]);
        load_square(nx, SQ_INV, inv);
        #pragma unroll
        for (int c = 0; c < VC; c++)
            stw4(u_s + (c * 16 + lr) * TS + w * 16 + g * 4, VP,
                 GEN ? -u[c] : u[c]);
        lds_barrier();
        // results and the next state
        #pragma unroll
        for (int j = 0; j < 2; j++)
            #pragma unroll
            for (int c = 0; c < VC; c++) {
                const Wide<T> b = wide_at(u_s, c, j);
                ao[c] = mma(GEN ? aqe[j] : aqk[j], b, ao[c]);
                #pragma unroll
                for (int x = 0; x < NS; x++)
                    S[x][c] = mma(GEN ? ef[x][j] : kf[x][j], b, S[x][c]);
                if (GEN) {
                    const Frag<T> v = frag8(vb + (c * 16 + lr) * TS + j * 32
                                            + g * 8);
                    #pragma unroll
                    for (int x = 0; x < NS; x++)
                        S[x][c] = mma(kf[x][j], v, S[x][c]);
                }
            }
        load_square(nx, GEN ? SQ_QE : SQ_QK, GEN ? aqe : aqk);
        load_k(nx);
        #pragma unroll
        for (int c = 0; c < VC; c++) {
            const int v = v0 + c * 16 + lr;
            #pragma unroll
            for (int i = 0; i < 4; i++) {
                const int t = w * 16 + g * 4 + i;
                if (t < n && v < V)
                    o[((int64_t)(t0 + t) * H + h) * V + v] = ao[c][i];
            }
        }
    }
    #pragma unroll
    for (int x = 0; x < NS; x++)
        #pragma unroll
        for (int c = 0; c < VC; c++)
            #pragma unroll
            for (int i = 0; i < 4; i++) {
                const int d = (w + x * 4) * 16 + g * 4 + i;
                const int v = v0 + c * 16 + lr;
                if (d < D && v < V) St[(int64_t)d * V + v] = S[x][c][i];
            }
}

// key channels of the chunk kernels' tiles
static int delta_tiles(int D) { return D <= 64 ? 64 : D <= 128 ? 128 : 256; }

extern "C" int64_t delta_scratch_floats(int gen, int n_chunks, int H, int D)
{
    const int64_t dp = delta_tiles(D);
    return (int64_t)n_chunks * H * ((gen ? 4 : 3) * CH * dp
                                    + (gen ? 4 : 2) * CH * CH + dp);
}

struct Scan {
    float* o; float* scr; float* state;
    const int* slot; const int* pos; const int* chunks; int n_chunks;
    const int* seqs; int n_seqs;
    hipStream_t stream;
};

template <typename T, int NS, int VC, bool GEN, bool VEC>
static void scan_go(const DeltaIn<T>& in, const Scan& a)
{
    constexpr int W = VC * 16, PAD = 16 / sizeof(T), es = sizeof(T);
    constexpr int NT = Terms<T>::N;
    constexpr int lds = es * W * (NT * (NS * 64 + PAD)
                                  + (2 * NT + (GEN ? 2 : 1)) * (CH + PAD));
    static bool once = false;
    if (!once) {
        (void)hipFuncSetAttribute(
            (const void*)k_delta_scan<T, NS, VC, GEN, VEC>,
            hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
        once = true;
    }
    const int heads = (a.n_seqs * in.H + XCDS - 1) / XCDS * XCDS;
    k_delta_scan<T, NS, VC, GEN, VEC>
        <<<heads * ((in.V + W - 1) / W), 256, lds, a.stream>>>(
            a.o, a.scr, in, a.state, a.slot, a.pos, a.chunks, a.seqs,
            a.n_seqs);
}

template <typename T, bool GEN, int NS, bool VEC>
static void prep_go(const DeltaIn<T>& in, const Scan& a)
{
    constexpr int part = ((GEN ? 6 : 7) * CH * DS + 4 * DB) * 4;
    constexpr int solve = 2 * CH * AS * 4;
    static bool once = false;
    if (!once) {
        (void)hipFuncSetAttribute(
            (const void*)k_delta_prep<T, GEN, NS * 64, VEC>,
            hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
        once = true;
    }
    k_delta_prep<T, GEN, NS * 64, VEC>
        <<<dim3(a.n_chunks, in.H), 256, part > solve ? part : solve,
           a.stream>>>(a.scr, in, a.chunks);
}

template <typename T, bool GEN, int NS>
static int chunks_go(const DeltaIn<T>& in, const Scan& a)
{
    static_assert(Unit<T, GEN, NS * 64>::floats
                  == (GEN ? 4 : 3) * CH * NS * 64 + (GEN ? 4 : 2) * CH * CH
                     + NS * 64, "scratch");
    const int D = in.D, V = in.V;
    if (D % 8 == 0 && in.oq % 8 == 0 && in.ok % 8 == 0 && in.oa % 8 == 0
        && in.ld % 8 == 0)
        prep_go<T, GEN, NS, true>(in, a);
    else prep_go<T, GEN, NS, false>(in, a);
    // wide strips share the loads of the factors, narrow ones fill the chip
    constexpr int WIDE = NS < 4 ? 2 : 1;
    const bool wide = (int64_t)a.n_seqs * in.H * ((V + 31) / 32) >= 256;
    if (V % 4 || in.ov % 4 || in.ld % 4) scan_go<T, NS, 1, GEN, false>(in, a);
    else if (wide) scan_go<T, NS, WIDE, GEN, true>(in, a);
    else scan_go<T, NS, 1, GEN, true>(in, a);
    return (int)hipGetLastError();
}

template <typename T, bool GEN>
static int chunks_for(const DeltaIn<T>& in, const Scan& a)
{
    if (in.D < 1 || in.V < 1 || in.D > 256) return (int)hipErrorInvalidValue;
    const int dp = delta_tiles(in.D);
    return dp == 64 ? chunks_go<T, GEN, 1>(in, a)
           : dp == 128 ? chunks_go<T, GEN, 2>(in, a)
                       : chunks_go<T, GEN, 4>(in, a);
}

// Portions of whole sequences in chunks of 64 rows.  chunks int32 [n, 2]
// (first row, rows), a sequence's chunks in a run; seqs int32 [m, 2] (first
// chunk, chunks); D <= 256.
extern "C" int delta_chunks(
    int f32, int gen, void* o, void* scr, const void* x, int64_t ld, int oq,
    int ok, int ov, int oa, const void* qs, const void* ks, int sld,
    const void* decay, const void* beta, const void* a_bias, void* state,
    const void* slot, const void* pos, const void* chunks, int n_chunks,
    const void* seqs, int n_seqs, int H, int G, int D, int V,
    hipStream_t stream)
{
    const Scan a{(float*)o, (float*)scr, (float*)state, (const int*)slot,
                 (const int*)pos, (const int*)chunks, n_chunks,
                 (const int*)seqs, n_seqs, stream};
    #define DC_GO(T, GEN) chunks_for<T, GEN>(DELTA_IN(T), a)
    if (f32) return gen ? DC_GO(float, true) : DC_GO(float, false);
    return gen ? DC_GO(bf16, true) : DC_GO(bf16, false);
    #undef DC_GO
}
