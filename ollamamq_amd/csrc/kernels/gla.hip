// gfx950 gated linear attention: per head a [D, V] fp32 state with
//   S_t = diag(alpha_t) S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t,
// alpha_t = sigmoid(z_t)^(1/tau) per key channel, z = a2 u + b from the
// low-rank projection u.  The recurrence is fp32 throughout, on the fp32
// matrix cores in chunks, in both element types of the surrounding model.
//
// * k_gla_step: a token at a time (decode, portions of a few tokens), with
//   the head norm and the output gate in the same kernel.
// * k_gla_prep / k_gla_scan / k_gla_out: chunks of 64 tokens.  With b the
//   running sum of log alpha inside a chunk,
//     o_i = (q_i e^{b_i}) S_0 + sum_{j<=i} (sum_d q_id k_jd e^{b_id-b_jd}) v_j
//     S'  = diag(e^{b_64}) S_0 + sum_j (k_j e^{b_64-b_j}) v_j^T.
//   prep makes the three decayed factors for all chunks at once; scan walks
//   a sequence's chunks with the state in registers.  No exponent is ever
//   positive: sums are kept per 16-token part, and a pair of parts is joined
//   by the decay across the parts between them.
// A sequence starts where its position is 0: the state is then taken as
// zero and whatever the slot held is ignored.
#include "tile_mma.h"

struct GlaIn {            // one row of the fused projection
    int64_t ld;           // row stride
    int oq, ok, ov, og, ou;   // column offsets of q, k, v, gate, low rank
    int rank;
};

// log(sigmoid(z)) / tau; the error of log(1 + e) is absolute, like that of
// any exponent near zero
DEV float log_alpha(float z, float inv_tau) {
    return (fminf(z, 0.f) - __logf(1.f + __expf(-fabsf(z)))) * inv_tau;
}
DEV float silu(float x) { return x / (1.f + __expf(-x)); }

template <typename T, int VEC>
__global__ __launch_bounds__(256, 2) void k_gla_step(
    T* __restrict__ out,                // [T, H*V]
    const T* __restrict__ p, GlaIn in,
    const T* __restrict__ a2, const float* __restrict__ a2_b,
    const float* __restrict__ norm_w,
    float* __restrict__ state,          // [slots, H, D, V]
    const int* __restrict__ slot, const int* __restrict__ pos,
    const int* __restrict__ spans,      // [n, 2] first row, rows; null: 1 row
    int H, int D, int V, float scale, float inv_tau, float eps,
    int frag)                           // layout of out
{
    const int h = blockIdx.y, tid = threadIdx.x;
    const int t0 = spans ? spans[blockIdx.x * 2] : blockIdx.x;
    const int nt = spans ? spans[blockIdx.x * 2 + 1] : 1;
    const int nv = min(V / VEC, 256);   // threads across a state row
    const int RG = 256 / nv;            // state rows in flight
    const int rg = tid / nv;
    extern __shared__ __attribute__((aligned(16))) float sm[];
    float* q_s = sm;                    // [D]
    float* k_s = q_s + D;
    float* a_s = k_s + D;
    float* o_s = a_s + D;               // [RG][V]
    float* r_s = o_s + RG * V;          // [4]
    float* Sh = state + ((int64_t)slot[t0] * H + h) * D * V;
    const int vt0 = rg < RG ? tid % nv : V;
    bool fresh = pos[t0] == 0;
    // state rows in flight: the first are asked for before the decays are
    // worked out, then always one group ahead
    constexpr int PF = 8;
    float nxt[PF][VEC];
    auto ahead = [&](const float* S, int d0) {
        #pragma unroll
        for (int j = 0; j < PF; j++) {
            const int d = d0 + j * RG;
            if (!fresh && d < D) ldv<VEC>(S + (int64_t)d * V, nxt[j]);
            else
                #pragma unroll
                for (int i = 0; i < VEC; i++) nxt[j][i] = 0.f;
        }
    };
    for (int t = t0; t < t0 + nt; ++t) {
        const T* row = p + (int64_t)t * in.ld;
        if (vt0 * VEC < V) ahead(Sh + vt0 * VEC, rg);
        for (int d = tid; d < D; d += 256) {
            const int c = h * D + d;
            q_s[d] = ldf(row + in.oq + c) * scale;
            k_s[d] = ldf(row + in.ok + c);
            float z = a2_b[c];
            for (int r = 0; r < in.rank; r++)
                z += ldf(a2 + (int64_t)c * in.rank + r)
                     * ldf(row + in.ou + r);
            a_s[d] = __expf(log_alpha(z, inv_tau));
        }
        __syncthreads();
        for (int vt = vt0; vt * VEC < V; vt += nv) {
            float* S = Sh + vt * VEC;
            float v[VEC], acc[VEC] = {};
            if (vt != vt0) ahead(S, rg);
            ldv<VEC>(row + in.ov + h * V + vt * VEC, v);
            for (int d0 = rg; d0 < D; d0 += RG * PF) {
                float s[PF][VEC];
                #pragma unroll
                for (int j = 0; j < PF; j++)
                    #pragma unroll
                    for (int i = 0; i < VEC; i++) s[j][i] = nxt[j][i];
                if (d0 + RG * PF < D) ahead(S, d0 + RG * PF);
                #pragma unroll
                for (int j = 0; j < PF; j++) {
                    const int d = d0 + j * RG;
                    if (d >= D) break;
                    #pragma unroll
                    for (int i = 0; i < VEC; i++) {
                        s[j][i] = a_s[d] * s[j][i] + k_s[d] * v[i];
                        acc[i] += q_s[d] * s[j][i];
                    }
                    stv<VEC>(S + (int64_t)d * V, s[j]);
                }
            }
            stv<VEC>(o_s + rg * V + vt * VEC, acc);
        }
        fresh = false;
        __syncthreads();
        float sq = 0.f;
        for (int c = tid; c < V; c += 256) {
            float o = 0.f;
            for (int r = 0; r < RG; r++) o += o_s[r * V + c];
            o_s[c] = o;                 // only this thread reads column c
            sq += o * o;
        }
        sq = wave_sum(sq);
        if ((tid & 63) == 0) r_s[tid >> 6] = sq;
        __syncthreads();
        const float ms = ((r_s[0] + r_s[1]) + (r_s[2] + r_s[3])) / V;
        const float rs = 1.f / sqrtf(ms + eps);
        for (int c = tid; c < V; c += 256)
            stf(out + (frag ? frag_row_off(t, h * V + c, H * V)
                            : ((int64_t)t * H + h) * V + c),
                o_s[c] * rs * norm_w[c]
                    * silu(ldf(row + in.og + h * V + c)));
        __syncthreads();
    }
}

extern "C" int gla_step(
    int f32, void* out, const void* p, int64_t ld, int oq, int ok, int ov,
    int og, int ou, int rank, const void* a2, const void* a2_b,
    const void* norm_w, void* state, const void* slot, const void* pos,
    const void* spans, int n, int H, int D, int V, float scale,
    float inv_tau, float eps, int frag, hipStream_t stream)
{
    // a vector load of v needs aligned columns
    const bool v4 = V % 4 == 0 && ov % 4 == 0 && ld % 4 == 0;
    GlaIn in{ld, oq, ok, ov, og, ou, rank};
    const int nv = v4 ? V / 4 : V;
    const int rg = nv < 256 ? 256 / nv : 1;
    const int64_t lds = ((int64_t)3 * D + (int64_t)rg * V + 4) * 4;
    if (D < 1 || V < 1 || rank < 1 || lds > 64 * 1024)
        return (int)hipErrorInvalidValue;
    dim3 grid(n, H);
    #define GS_GO(T, VV)                                                   \
        k_gla_step<T, VV><<<grid, 256, lds, stream>>>(                     \
            (T*)out, (const T*)p, in, (const T*)a2, (const float*)a2_b,    \
            (const float*)norm_w, (float*)state, (const int*)slot,         \
            (const int*)pos, (const int*)spans, H, D, V, scale, inv_tau,   \
            eps, frag)
    if (f32) { if (v4) GS_GO(float, 4); else GS_GO(float, 1); }
    else { if (v4) GS_GO(bf16, 4); else GS_GO(bf16, 1); }
    #undef GS_GO
    return (int)hipGetLastError();
}

// ---- chunks --------------------------------------------------------------
#define CH 64             // tokens of a chunk
#define SUB 16            // tokens of a part
#define DB 32             // key channels of a prep pass
#define DS (DB + 1)       // LDS row stride
// largest sum of decay inside a part for which the part's own triangle may
// be factored (e^{b_i} e^{-b_j}); beyond it the pairs are taken one by one
#define SAFE 20.f

// scratch per (chunk, head): qd [64][Dp], kd^T [Dp][64], A [64][64], eb [Dp]
DEV int64_t gla_unit(int Dp) {
    return (int64_t)2 * CH * Dp + CH * CH + Dp;
}

// Wave w owns part w of the chunk.  z comes off the matrix cores with a
// channel on a lane and four tokens in its registers, so the running sum
// over the part is three adds and two cross-lane steps; only the factors
// that other lanes need as matrix operands go through LDS.
template <typename T>
__global__ __launch_bounds__(256) void k_gla_prep(
    float* __restrict__ scr, const T* __restrict__ p, GlaIn in,
    const T* __restrict__ a2, const float* __restrict__ a2_b,
    const int* __restrict__ chunks,     // [n, 2] first row, rows
    int H, int D, int Dp, float scale, float inv_tau, int vec)
{
    const int h = blockIdx.y, tid = threadIdx.x;
    const int lane = tid & 63, w = tid >> 6;
    const int lr = lane & 15, g = lane >> 4;
    const int t0 = chunks[blockIdx.x * 2], n = chunks[blockIdx.x * 2 + 1];
    const int R4 = (in.rank + 3) & ~3, RS = R4 + 1;
    float* qd = scr + ((int64_t)blockIdx.x * H + h) * gla_unit(Dp);
    float* kdt = qd + CH * Dp;
    float* Ao = kdt + CH * Dp;
    float* eb = Ao + CH * CH;
    extern __shared__ __attribute__((aligned(16))) float sm[];
    float* q_s = sm;                    // [64][DS] scaled q
    float* k_s = q_s + CH * DS;         // k, or k e^{-b}
    float* b_s = k_s + CH * DS;         // running log decay inside a part
    float* qe_s = b_s + CH * DS;        // q e^{b}
    float* ke_s = qe_s + CH * DS;       // k e^{part total - b}
    float* et_s = ke_s + CH * DS;       // [4][DB] e^{part total}
    float* w_s = et_s + 4 * DB;         // [DB][RS] rows of a2
    float* u_s = w_s + DB * RS;         // [64][RS]

    for (int i = tid; i < CH * R4; i += 256) {
        const int t = i / R4, r = i % R4;
        u_s[t * RS + r] = t < n && r < in.rank
            ? ldf(p + (int64_t)(t0 + t) * in.ld + in.ou + r) : 0.f;
    }
    // of the six tiles below the diagonal (1,0) (2,1) (3,2) (2,0) (3,1)
    // (3,0) this wave makes numbers w and w + 4
    const int ti[6] = {1, 2, 3, 2, 3, 3}, tj[6] = {0, 1, 2, 0, 1, 0};
    f32x4 diag = {}, off[2] = {};

    for (int d0 = 0; d0 < Dp; d0 += DB) {
        __syncthreads();
        for (int i = tid; i < DB * R4; i += 256) {
            const int d = i / R4, r = i % R4;
            w_s[d * RS + r] = d0 + d < D && r < in.rank
                ? ldf(a2 + (int64_t)(h * D + d0 + d) * in.rank + r) : 0.f;
        }
        #pragma unroll
        for (int x = 0; x < 2; x++) {       // 16 tokens x 32 channels by fours
            const int i = lane + x * 64;
            const int t = w * SUB + (i >> 3), d = (i & 7) * 4;
            const T* row = p + (int64_t)(t0 + t) * in.ld + h * D + d0 + d;
            float q4[4] = {}, k4[4] = {};
            if (t < n) {
                if (vec) {
                    if (d0 + d < D) {
                        ldv<4>(row + in.oq, q4);
                        ldv<4>(row + in.ok, k4);
                    }
                } else
                    for (int e = 0; e < 4; e++)
                        if (d0 + d + e < D) {
                            q4[e] = ldf(row + in.oq + e);
                            k4[e] = ldf(row + in.ok + e);
                        }
            }
            #pragma unroll
            for (int e = 0; e < 4; e++) {
                q_s[t * DS + d + e] = q4[e] * scale;
                k_s[t * DS + d + e] = k4[e];
            }
        }
        __syncthreads();
        f32x4 qe[2], ke[2];
        bool safe = true;
        float b[2][4];
        #pragma unroll
        for (int x = 0; x < 2; x++) {
            f32x4 z = {};
            for (int r = g; r < R4; r += 4)
                z = __builtin_amdgcn_mfma_f32_16x16x4f32(
                    u_s[(w * SUB + lr) * RS + r],
                    w_s[(x * 16 + lr) * RS + r], z, 0, 0, 0);
            const int d = x * 16 + lr;
            const bool on = d0 + d < D;
            const float bias = on ? a2_b[h * D + d0 + d] : 0.f;
            float run = 0.f;
            #pragma unroll
            for (int i = 0; i < 4; i++) {
                const int t = w * SUB + g * 4 + i;
                if (on && t < n) run += log_alpha(z[i] + bias, inv_tau);
                b[x][i] = run;
            }
            float inc = run;                // over the lanes' four-token runs
            const float u1 = __shfl_up(inc, 16, 64);
            if (g >= 1) inc += u1;
            const float u2 = __shfl_up(inc, 32, 64);
            if (g >= 2) inc += u2;
            float exc = __shfl_up(inc, 16, 64);
            if (g == 0) exc = 0.f;
            const float tot = __shfl(inc, 48 + lr, 64);
            safe = safe && tot > -SAFE;
            #pragma unroll
            for (int i = 0; i < 4; i++) {
                b[x][i] += exc;
                const int o = (w * SUB + g * 4 + i) * DS + d;
                qe[x][i] = q_s[o] * __expf(b[x][i]);
                ke[x][i] = k_s[o] * __expf(tot - b[x][i]);
                qe_s[o] = qe[x][i];
                ke_s[o] = ke[x][i];
            }
            if (g == 0) et_s[w * DB + d] = __expf(tot);
        }
        safe = __all(safe);
        #pragma unroll
        for (int x = 0; x < 2; x++)
            #pragma unroll
            for (int i = 0; i < 4; i++) {
                const int o = (w * SUB + g * 4 + i) * DS + x * 16 + lr;
                if (safe) k_s[o] *= __expf(-b[x][i]);
                else b_s[o] = b[x][i];
            }
        __syncthreads();
        // factors that meet the state
        #pragma unroll
        for (int x = 0; x < 2; x++) {
            const int d = x * 16 + lr;
            if (d0 + d >= Dp) continue;
            float before = 1.f, after = 1.f;
            for (int s = 0; s < w; s++) before *= et_s[s * DB + d];
            for (int s = w + 1; s < 4; s++) after *= et_s[s * DB + d];
            #pragma unroll
            for (int i = 0; i < 4; i++)
                qd[(w * SUB + g * 4 + i) * Dp + d0 + d] = qe[x][i] * before;
            *reinterpret_cast<f32x4*>(
                kdt + (int64_t)(d0 + d) * CH + w * SUB + g * 4) =
                ke[x] * after;
            if (w == 3 && g == 0)
                eb[d0 + d] = before * et_s[3 * DB + d];
        }
        // tiles below the diagonal
        #pragma unroll
        for (int x = 0; x < 2; x++) {
            const int id = w + x * 4;
            if (id >= 6) continue;
            const int I = ti[id], J = tj[id];
            #pragma unroll
            for (int d = 0; d < DB; d += 4) {
                float a = qe_s[(I * SUB + lr) * DS + d + g];
                for (int s = J + 1; s < I; s++) a *= et_s[s * DB + d + g];
                off[x] = __builtin_amdgcn_mfma_f32_16x16x4f32(
                    a, ke_s[(J * SUB + lr) * DS + d + g], off[x], 0, 0, 0);
            }
        }
        // the part's own triangle
        if (safe) {
            #pragma unroll
            for (int d = 0; d < DB; d += 4) {
                const int o = (w * SUB + lr) * DS + d + g;
                diag = __builtin_amdgcn_mfma_f32_16x16x4f32(
                    qe_s[o], k_s[o], diag, 0, 0, 0);
            }
        } else {
            // lane: column lr (the key), rows g*4 + i (the query)
            for (int d = 0; d < DB; d++) {
                const int oj = (w * SUB + lr) * DS + d;
                const float kj = k_s[oj], bj = b_s[oj];
                #pragma unroll
                for (int i = 0; i < 4; i++) {
                    const int oi = (w * SUB + g * 4 + i) * DS + d;
                    diag[i] += q_s[oi] * kj
                               * __expf(fminf(b_s[oi] - bj, 0.f));
                }
            }
        }
    }
    #pragma unroll
    for (int i = 0; i < 4; i++)
        Ao[(w * SUB + g * 4 + i) * CH + w * SUB + lr] =
            lr <= g * 4 + i ? diag[i] : 0.f;
    #pragma unroll
    for (int x = 0; x < 2; x++) {
        const int id = w + x * 4;
        if (id >= 6) continue;
        #pragma unroll
        for (int i = 0; i < 4; i++)
            Ao[(ti[id] * SUB + g * 4 + i) * CH + tj[id] * SUB + lr] =
                off[x][i];
    }
}

// A sequence's chunks in order, one block per 16*VC value columns, the state
// in registers (NS: 16-row tiles per wave, D <= 64 * NS).  Only the state
// and v go through LDS; every other operand belongs to one wave and comes
// straight from memory, loaded while the matrix cores work on what was
// loaded before.
template <typename T, int NS, int VC>
__global__ __launch_bounds__(256) void k_gla_scan(
    float* __restrict__ o,              // [rows, H, V]
    const float* __restrict__ scr, const T* __restrict__ p, GlaIn in,
    float* __restrict__ state,
    const int* __restrict__ slot, const int* __restrict__ pos,
    const int* __restrict__ chunks,     // [n, 2]
    const int* __restrict__ seqs,       // [m, 2] first chunk, chunks
    int row_base,                       // first row of o
    int H, int D, int Dp, int V)
{
    constexpr int W = VC * 16, WS = W + (W % 64 == 16 ? 0 : 16);
    constexpr int NQ = NS * 4;          // 16-channel steps over D
    constexpr int NV = CH * W / 256;    // elements of v a thread
    const int h = blockIdx.y, v0 = blockIdx.z * W, tid = threadIdx.x;
    const int lane = tid & 63, w = tid >> 6;
    const int lr = lane & 15, g = lane >> 4;
    const int c0 = seqs[blockIdx.x * 2], nc = seqs[blockIdx.x * 2 + 1];
    const int first = chunks[c0 * 2];
    float* St = state + ((int64_t)slot[first] * H + h) * D * V;
    extern __shared__ __attribute__((aligned(16))) float sm[];
    float* S_s = sm;                    // [Dp][WS]
    float* v_s = S_s + Dp * WS;         // [64][WS]

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

    // operands in flight; a lane's k runs in fours, the same for both sides
    f32x4 q4[NQ], a4[4], k4[NS][4], e4[NS];
    float vv[NV];
    auto unit = [&](int ci) {
        return scr + ((int64_t)ci * H + h) * gla_unit(Dp);
    };
    auto load_qa = [&](int ci) {
        const float* qr = unit(ci) + (w * 16 + lr) * Dp + g * 4;
        #pragma unroll
        for (int d = 0; d < NQ; d++)
            q4[d] = d * 16 < Dp
                ? *reinterpret_cast<const f32x4*>(qr + d * 16) : f32x4{};
        const float* Ar = unit(ci) + 2 * CH * Dp + (w * 16 + lr) * CH + g * 4;
        #pragma unroll
        for (int j = 0; j < 4; j++)
            a4[j] = j <= w
                ? *reinterpret_cast<const f32x4*>(Ar + j * 16) : f32x4{};
    };
    auto load_k = [&](int ci) {
        const float* kd = unit(ci) + CH * Dp;
        const float* eb = unit(ci) + 2 * CH * Dp + CH * CH;
        #pragma unroll
        for (int x = 0; x < NS; x++) {
            const int d = (w + x * 4) * 16;
            const bool in_d = d < Dp;
            e4[x] = in_d ? *reinterpret_cast<const f32x4*>(eb + d + g * 4)
                         : f32x4{};
            #pragma unroll
            for (int t = 0; t < 4; t++)
                k4[x][t] = in_d ? *reinterpret_cast<const f32x4*>(
                    kd + (int64_t)(d + lr) * CH + t * 16 + g * 4) : f32x4{};
        }
    };
    auto load_v = [&](int ci) {
        const int t0 = chunks[ci * 2], n = chunks[ci * 2 + 1];
        #pragma unroll
        for (int x = 0; x < NV; x++) {
            const int i = tid + x * 256, t = i / W, c = i % W;
            vv[x] = t < n && v0 + c < V
                ? ldf(p + (int64_t)(t0 + t) * in.ld + in.ov + h * V + v0 + c)
                : 0.f;
        }
    };
    load_v(c0);
    load_qa(c0);
    load_k(c0);

    for (int ci = c0; ci < c0 + nc; ++ci) {
        const int t0 = chunks[ci * 2], n = chunks[ci * 2 + 1];
        const int nx = min(ci + 1, c0 + nc - 1);
        #pragma unroll
        for (int x = 0; x < NV; x++) {
            const int i = tid + x * 256;
            v_s[(i / W) * WS + i % W] = vv[x];
        }
        #pragma unroll
        for (int x = 0; x < NS; x++) {
            const int d0 = (w + x * 4) * 16;
            if (d0 < Dp)
                #pragma unroll
                for (int c = 0; c < VC; c++)
                    #pragma unroll
                    for (int i = 0; i < 4; i++)
                        S_s[(d0 + g * 4 + i) * WS + c * 16 + lr] =
                            S[x][c][i];
        }
        __syncthreads();
        load_v(nx);
        // state: needs only v and registers
        #pragma unroll
        for (int x = 0; x < NS; x++) {
            #pragma unroll
            for (int c = 0; c < VC; c++) S[x][c] *= e4[x];
            #pragma unroll
            for (int t = 0; t < 4; t++)
                #pragma unroll
                for (int e = 0; e < 4; e++)
                    #pragma unroll
                    for (int c = 0; c < VC; c++)
                        S[x][c] = __builtin_amdgcn_mfma_f32_16x16x4f32(
                            k4[x][t][e],
                            v_s[(t * 16 + g * 4 + e) * WS + c * 16 + lr],
                            S[x][c], 0, 0, 0);
        }
        load_k(nx);
        // o tile of this wave's 16 tokens
        f32x4 acc[VC] = {};
        #pragma unroll
        for (int d = 0; d < NQ; d++)
            if (d * 16 < Dp)
                #pragma unroll
                for (int e = 0; e < 4; e++)
                    #pragma unroll
                    for (int c = 0; c < VC; c++)
                        acc[c] = __builtin_amdgcn_mfma_f32_16x16x4f32(
                            q4[d][e],
                            S_s[(d * 16 + g * 4 + e) * WS + c * 16 + lr],
                            acc[c], 0, 0, 0);
        #pragma unroll
        for (int j = 0; j < 4; j++)
            if (j <= w)
                #pragma unroll
                for (int e = 0; e < 4; e++)
                    #pragma unroll
                    for (int c = 0; c < VC; c++)
                        acc[c] = __builtin_amdgcn_mfma_f32_16x16x4f32(
                            a4[j][e],
                            v_s[(j * 16 + g * 4 + e) * WS + c * 16 + lr],
                            acc[c], 0, 0, 0);
        load_qa(nx);
        #pragma unroll
        for (int c = 0; c < VC; c++)
            #pragma unroll
            for (int i = 0; i < 4; i++) {
                const int t = w * 16 + g * 4 + i, v = v0 + c * 16 + lr;
                if (t < n && v < V)
                    o[((int64_t)(t0 - row_base + t) * H + h) * V + v] =
                        acc[c][i];
            }
        __syncthreads();
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

// head norm and gate, one wave per (token, head)
template <typename T, int VEC>
__global__ __launch_bounds__(256) void k_gla_out(
    T* __restrict__ out, const float* __restrict__ o,
    const T* __restrict__ p, GlaIn in, const float* __restrict__ norm_w,
    int row_base, int64_t n, int H, int V, float eps)
{
    const int64_t u = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    const int lane = threadIdx.x & 63;
    if (u >= n) return;
    const int64_t t = u / H;
    const int h = (int)(u % H);
    const float* src = o + u * V;
    float sq = 0.f;
    float x[VEC], gt[VEC], nw[VEC];
    const bool one = V <= 64 * VEC;         // the row fits the wave
    for (int c = lane * VEC; c < V; c += 64 * VEC) {
        ldv<VEC>(src + c, x);
        #pragma unroll
        for (int i = 0; i < VEC; i++) sq += x[i] * x[i];
    }
    const float rs = 1.f / sqrtf(wave_sum(sq) / V + eps);
    const T* gr = p + (row_base + t) * in.ld + in.og + h * V;
    T* dst = out + ((row_base + t) * H + h) * V;
    for (int c = lane * VEC; c < V; c += 64 * VEC) {
        if (!one) ldv<VEC>(src + c, x);
        ldv<VEC>(gr + c, gt);
        ldv<VEC>(norm_w + c, nw);
        #pragma unroll
        for (int i = 0; i < VEC; i++) x[i] *= rs * nw[i] * silu(gt[i]);
        stv<VEC>(dst + c, x);
    }
}

extern "C" int64_t gla_scratch_floats(int n_chunks, int H, int D)
{
    const int Dp = (D + 15) & ~15;
    return (int64_t)n_chunks * H * (2 * CH * Dp + CH * CH + Dp);
}

// Portions of whole sequences in chunks of 64 rows.  chunks int32 [n, 2]
// (first row, rows), a sequence's chunks in a run; seqs int32 [m, 2] (first
// chunk, chunks); D <= 512, rank <= 256.  Rows row_base .. row_base + rows - 1 are covered.
extern "C" int gla_chunks(
    int f32, void* out, void* scr, void* o_scr, const void* p, int64_t ld,
    int oq, int ok, int ov, int og, int ou, int rank, const void* a2,
    const void* a2_b, const void* norm_w, void* state, const void* slot,
    const void* pos, const void* chunks, int n_chunks, const void* seqs,
    int n_seqs, int row_base, int rows, int H, int D, int V, float scale,
    float inv_tau, float eps, hipStream_t stream)
{
    if (D < 1 || V < 1 || rank < 1 || D > 512 || rank > 256)
        return (int)hipErrorInvalidValue;
    GlaIn in{ld, oq, ok, ov, og, ou, rank};
    const int Dp = (D + 15) & ~15;
    const int rs = ((rank + 3) & ~3) + 1;
    const int lds_a = (5 * CH * DS + 4 * DB + (CH + DB) * rs) * 4;
    // wider column tiles re-read the factors less; narrow ones fill the chip
    const int vc = (int64_t)n_seqs * H * ((V + 31) / 32) >= 512
                   && Dp <= 256 ? 2 : 1;
    const int vec = D % 4 == 0 && oq % 4 == 0 && ok % 4 == 0 && ld % 4 == 0;
    const bool vout = V % 4 == 0 && og % 4 == 0 && ld % 4 == 0;
    const int ws = vc == 1 ? 16 : 48;
    const int lds_b = (Dp + CH) * ws * 4;
    if (lds_a > 160 * 1024 || lds_b > 160 * 1024)
        return (int)hipErrorInvalidValue;
    dim3 ga(n_chunks, H), gb(n_seqs, H, (V + vc * 16 - 1) / (vc * 16));
    const int64_t units = (int64_t)rows * H;
    const int gc = (int)((units + 3) / 4);
    #define GC_SCAN(T, NS, VC)                                             \
        do {                                                               \
            (void)hipFuncSetAttribute(                                     \
                (const void*)k_gla_scan<T, NS, VC>,                        \
                hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);   \
            k_gla_scan<T, NS, VC><<<gb, 256, lds_b, stream>>>(             \
                (float*)o_scr, (const float*)scr, (const T*)p, in,         \
                (float*)state, (const int*)slot, (const int*)pos,          \
                (const int*)chunks, (const int*)seqs, row_base, H, D, Dp,  \
                V);                                                        \
        } while (0)
    #define GC_NS(T, VC)                                                   \
        do {                                                               \
            if (Dp <= 64) GC_SCAN(T, 1, VC);                               \
            else if (Dp <= 128) GC_SCAN(T, 2, VC);                         \
            else if (Dp <= 256) GC_SCAN(T, 4, VC);                         \
            else GC_SCAN(T, 8, VC);                                        \
        } while (0)
    #define GC_OUT(T, VV)                                                  \
        k_gla_out<T, VV><<<gc, 256, 0, stream>>>(                          \
            (T*)out, (const float*)o_scr, (const T*)p, in,                 \
            (const float*)norm_w, row_base, units, H, V, eps)
    #define GC_TYPE(T)                                                     \
        do {                                                               \
            (void)hipFuncSetAttribute(                                     \
                (const void*)k_gla_prep<T>,                                \
                hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);   \
            k_gla_prep<T><<<ga, 256, lds_a, stream>>>(                     \
                (float*)scr, (const T*)p, in, (const T*)a2,                \
                (const float*)a2_b, (const int*)chunks, H, D, Dp, scale,   \
                inv_tau, vec);                                             \
            if (vc == 1) GC_NS(T, 1); else GC_NS(T, 2);                    \
            if (vout) GC_OUT(T, 4); else GC_OUT(T, 1);                     \
        } while (0)
    if (f32) GC_TYPE(float); else GC_TYPE(bf16);
    #undef GC_TYPE
    #undef GC_OUT
    #undef GC_NS
    #undef GC_SCAN
    return (int)hipGetLastError();
}
