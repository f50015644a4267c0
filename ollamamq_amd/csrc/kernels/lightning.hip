// gfx950 lightning attention: per head a [D, V] fp32 state with one decay,
//   S_t = r S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t,   q, k, v their columns in
// the fused projection, or the silu of them.  The state and everything that
// enters it beyond q, k and v is fp32: in bf16 models an fp32 operand of a
// matrix product goes through the bf16 matrix cores as the sum of two bf16
// terms.
//
// * k_lightning_step: a token at a time (decode, portions of a few tokens);
// * k_lightning_act / k_lightning_scan: chunks of 64 tokens.  Inside a chunk
//     o_i = r^(i+1) q_i S_0 + sum_{j<=i} r^(i-j) (q_i . k_j) v_j
//     S'  = r^n S_0 + sum_j k_j (r^(n-1-j) v_j)^T,
//   every factor a power of r between r^0 and r^64, from a table.  act makes
//   the padded rows of q, k and v once; scan walks a sequence's chunks with
//   the state in registers, a block per head and strip of value columns.
// The results o [T, H, V] are fp32; the norm and gate that follow are
// k_rms_gate or k_head_gate.  A sequence starts where its position is 0: the
// state is then taken as zero and whatever the slot held is ignored.
#include "tile_mma.h"

struct Cols { int q, k, v, act; };    // first columns in the projection
template <typename T> DEV float act_of(const Cols& at, float x) {
    return at.act ? silu_of<T>(x) : x;
}

#define CH 64                         // tokens of a chunk
#define PW (CH + 1)                   // powers per head

template <typename T, typename P, int VEC>
__global__ __launch_bounds__(256, 2) void k_lightning_step(
    float* __restrict__ o,              // [T, H, V]
    Rows<P> p, Cols at, const float* __restrict__ powers,   // [H, PW]
    float* __restrict__ state,          // [slots, H, D, V]
    const int* __restrict__ slot, const int* __restrict__ pos,
    const int* __restrict__ spans,      // [n, 2] first row, rows; null: 1 row
    int H, int D, int V, int VB)        // value columns of a block
{
    const int h = blockIdx.y, tid = threadIdx.x;
    const int v0 = blockIdx.z * VB, nc = min(VB, V - v0);
    const int t0 = spans ? spans[blockIdx.x * 2] : blockIdx.x;
    const int nt = spans ? spans[blockIdx.x * 2 + 1] : 1;
    const int nv = nc / VEC;            // threads across a state row
    const int RG = 256 / nv;            // state rows side by side
    const int rg = tid / nv;
    const bool on = rg < RG;
    const int vt = tid % nv * VEC;
    extern __shared__ __attribute__((aligned(16))) float sm[];
    float* q_s = sm;                    // [D]
    float* k_s = q_s + D;
    float* o_s = k_s + D;               // [RG][nc]
    const float r = powers[h * PW + 1];
    float* S = state + ((int64_t)slot[t0] * H + h) * D * V + v0 + vt;
    bool fresh = pos[t0] == 0;
    // state rows in flight: the first are asked for before q and k are
    // worked out, then always one group ahead
    constexpr int PF = 8;
    float nxt[PF][VEC];
    auto ahead = [&](int d0) {
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
        if (on) ahead(rg);
        for (int d = tid; d < D; d += 256) {
            float x;
            ldrow<1>(p, t, at.q + h * D + d, &x);
            q_s[d] = act_of<T>(at, x);
            ldrow<1>(p, t, at.k + h * D + d, &x);
            k_s[d] = act_of<T>(at, x);
        }
        __syncthreads();
        if (on) {
            float v[VEC], acc[VEC] = {};
            ldrow<VEC>(p, t, at.v + h * V + v0 + vt, v);
            #pragma unroll
            for (int i = 0; i < VEC; i++) v[i] = act_of<T>(at, v[i]);
            for (int d0 = rg; d0 < D; d0 += RG * PF) {
                float s[PF][VEC];
                #pragma unroll
                for (int j = 0; j < PF; j++)
                    #pragma unroll
                    for (int i = 0; i < VEC; i++) s[j][i] = nxt[j][i];
                if (d0 + RG * PF < D) ahead(d0 + RG * PF);
                #pragma unroll
                for (int j = 0; j < PF; j++) {
                    const int d = d0 + j * RG;
                    if (d >= D) break;
                    #pragma unroll
                    for (int i = 0; i < VEC; i++) {
                        s[j][i] = r * s[j][i] + k_s[d] * v[i];
                        acc[i] += q_s[d] * s[j][i];
                    }
                    stv<VEC>(S + (int64_t)d * V, s[j]);
                }
            }
            stv<VEC>(o_s + rg * nc + vt, acc);
        }
        fresh = false;
        __syncthreads();
        for (int c = tid; c < nc; c += 256) {
            float x = 0.f;
            for (int g = 0; g < RG; g++) x += o_s[g * nc + c];
            o[((int64_t)t * H + h) * V + v0 + c] = x;
        }
        __syncthreads();
    }
}

extern "C" int lightning_step(
    int f32, void* o, const void* p, int p32, int n_part,
    int64_t part_stride, int64_t ld, int oq, int ok, int ov, int act,
    const void* powers, void* state, const void* slot, const void* pos,
    const void* spans, int n, int H, int D, int V, hipStream_t stream)
{
    const bool v4 = V % 4 == 0 && ov % 4 == 0 && ld % 4 == 0
                    && part_stride % 4 == 0;
    if (D < 1 || V < 1 || D > 4096) return (int)hipErrorInvalidValue;
    // strips of 32 columns or more, narrower while there are few blocks
    int vb = V < 256 ? V : 256;
    while (v4 && vb > 32 && vb % 8 == 0
           && (int64_t)n * H * ((V + vb - 1) / vb) < 512) vb /= 2;
    const int nv = v4 ? vb / 4 : vb;
    // the last strip may be narrower, with more rows side by side
    const int lds = (2 * D + (256 / nv + 1) * vb + 1024) * 4;
    dim3 grid(n, H, (V + vb - 1) / vb);
    #define LS(T, P, VE)                                                   \
        k_lightning_step<T, P, VE><<<grid, 256, lds, stream>>>(            \
            (float*)o, Rows<P>{(const P*)p, n_part, part_stride, ld},      \
            Cols{oq, ok, ov, act}, (const float*)powers, (float*)state,         \
            (const int*)slot, (const int*)pos, (const int*)spans, H, D, V, \
            vb)
    #define LS_V(T, P) do { if (v4) LS(T, P, 4); else LS(T, P, 1); } while (0)
    if (f32) LS_V(float, float);
    else if (p32) LS_V(bf16, float);
    else LS_V(bf16, bf16);
    #undef LS_V
    #undef LS
    return (int)hipGetLastError();
}

// ---- chunks --------------------------------------------------------------

// a = q [H, rows, Dp], k [H, rows, Dp], v [H, rows, Vp], activated and filled
// up with zeros
template <typename T, typename P, int VEC>
__global__ __launch_bounds__(256) void k_lightning_act(
    T* __restrict__ a, Rows<P> p, Cols at, int row_base, int rows,
    int64_t total, int H, int D, int V, int Dp, int Vp)
{
    const int64_t N = (int64_t)H * (2 * Dp + Vp);
    for (int64_t i = (blockIdx.x * (int64_t)256 + threadIdx.x) * VEC;
         i < total; i += (int64_t)gridDim.x * 256 * VEC) {
        const int64_t t = i / N;
        int c = (int)(i - t * N), off = at.q, wide = D, pad = Dp;
        T* dst = a;
        if (c >= 2 * H * Dp) {
            c -= 2 * H * Dp;
            off = at.v, wide = V, pad = Vp;
            dst += (int64_t)2 * H * rows * Dp;
        } else if (c >= H * Dp) {
            c -= H * Dp;
            off = at.k;
            dst += (int64_t)H * rows * Dp;
        }
        const int h = c / pad, d = c % pad;
        float v[VEC] = {};
        if (d < wide) {
            ldrow<VEC>(p, row_base + t, off + h * wide + d, v);
            #pragma unroll
            for (int e = 0; e < VEC; e++) v[e] = act_of<T>(at, v[e]);
        }
        stv<VEC>(dst + ((int64_t)h * rows + t) * pad + d, v);
    }
}

template <typename T, int NS, int VC>
__global__ __launch_bounds__(256) void k_lightning_scan(
    float* __restrict__ o,              // [T, H, V]
    const T* __restrict__ a, const float* __restrict__ powers,
    float* __restrict__ state,
    const int* __restrict__ slot, const int* __restrict__ pos,
    const int* __restrict__ chunks,     // [n, 2] first row, rows
    const int* __restrict__ seqs,       // [m, 2] first chunk, chunks
    int row_base, int a_rows, int H, int D, int V, int Dp, int Vp)
{
    constexpr int W = VC * 16, PAD = 16 / sizeof(T), NT = Terms<T>::N;
    constexpr int DM = NS * 64, KS = DM + PAD, VS = W + PAD;
    constexpr int DQ = NS * 2;          // 32-channel steps over D
    constexpr int NK = NS * 2;          // 8-element pieces of k a thread
    constexpr int NV = (VC + 1) / 2;    // and of v
    const int h = blockIdx.y, v0 = blockIdx.z * W, tid = threadIdx.x;
    const int lane = tid & 63;
    const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int lr = lane & 15, g = lane >> 4;
    const int c0 = seqs[blockIdx.x * 2], nc = seqs[blockIdx.x * 2 + 1];
    // a sequence's rows follow one another: every chunk but the last is full
    const int first = chunks[c0 * 2];
    const int rows = (nc - 1) * CH + chunks[(c0 + nc - 1) * 2 + 1];
    const int64_t a0 = (int64_t)h * a_rows + first - row_base;
    const int64_t a_qk = (int64_t)H * a_rows * Dp;
    const T* aq = a + a0 * Dp;
    const T* ak = aq + a_qk;
    const T* av = a + 2 * a_qk + a0 * Vp + v0;
    float* St = state + ((int64_t)slot[first] * H + h) * D * V;
    extern __shared__ __attribute__((aligned(16))) char smem[];
    T* k_s = reinterpret_cast<T*>(smem);          // [CH][KS]
    T* v_s = k_s + CH * KS;                       // [CH][VS]
    T* d_s = v_s + CH * VS;                       // [NT][CH][VS] decayed v
    T* S_s = d_s + NT * CH * VS;                  // [NT][W][KS] state
    float* pw = reinterpret_cast<float*>(S_s + NT * W * KS);    // [PW]
    for (int i = tid; i < PW; i += 256) pw[i] = powers[h * PW + i];
    __syncthreads();

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
    // this lane's query is token w*16 + lr: its factors are the same in
    // every chunk
    const int me = w * 16 + lr;
    f32x4 fade[4];
    #pragma unroll
    for (int kt = 0; kt < 4; kt++)
        #pragma unroll
        for (int i = 0; i < 4; i++) {
            const int d = me - (kt * 16 + g * 4 + i);
            fade[kt][i] = d >= 0 ? pw[d] : 0.f;
        }
    const float fade0 = pw[me + 1];

    Frag<T> qf[DQ], kp[NK], vp[NV];
    float vw[NV];                       // factor of a piece of v
    // rows past the chunk's end repeat its last one and weigh nothing
    auto load_q = [&](int t0) {
        const T* r = aq + (int64_t)min(t0 + me, rows - 1) * Dp + g * 8;
        #pragma unroll
        for (int d = 0; d < DQ; d++)
            qf[d] = d * 32 < Dp ? frag8(r + d * 32) : frag_zero<T>();
    };
    auto load_kv = [&](int t0) {
        const int n = min(CH, rows - t0);
        #pragma unroll
        for (int j = 0; j < NK; j++) {
            const int u = tid + j * 256;
            const int t = u / (DM / 8), c = u % (DM / 8) * 8;
            kp[j] = c < Dp ? frag8(ak + (int64_t)(t0 + min(t, n - 1)) * Dp + c)
                           : frag_zero<T>();
        }
        #pragma unroll
        for (int j = 0; j < NV; j++) {
            const int u = tid + j * 256;
            const int t = u / (W / 8), c = u % (W / 8) * 8;
            vp[j] = frag_zero<T>();
            vw[j] = 0.f;
            if (t < n && v0 + c < Vp) {
                vp[j] = frag8(av + (int64_t)(t0 + t) * Vp + c);
                vw[j] = pw[n - 1 - t];
            }
        }
    };
    load_kv(0);
    load_q(0);

    for (int t0 = 0; t0 < rows; t0 += CH) {
        const int n = min(CH, rows - t0);
        const int nx = t0 + CH < rows ? t0 + CH : t0;
        #pragma unroll
        for (int j = 0; j < NK; j++) {
            const int u = tid + j * 256;
            *reinterpret_cast<Frag<T>*>(
                k_s + u / (DM / 8) * KS + u % (DM / 8) * 8) = kp[j];
        }
        #pragma unroll
        for (int j = 0; j < NV; j++) {
            const int u = tid + j * 256;
            const int t = u / (W / 8), c = u % (W / 8) * 8;
            if (t >= CH) continue;
            *reinterpret_cast<Frag<T>*>(v_s + t * VS + c) = vp[j];
            Frag<T> term[NT];
            #pragma unroll
            for (int e = 0; e < 8; e++) {
                T x[NT];
                Terms<T>::split(frag_get(vp[j], e) * vw[j], x);
                #pragma unroll
                for (int q = 0; q < NT; q++)
                    frag_set(term[q], e, ldf(&x[q]));
            }
            #pragma unroll
            for (int q = 0; q < NT; q++)
                *reinterpret_cast<Frag<T>*>(d_s + (q * CH + t) * VS + c) =
                    term[q];
        }
        #pragma unroll
        for (int x = 0; x < NS; x++) {
            const int d0 = (w + x * 4) * 16 + g * 4;
            #pragma unroll
            for (int c = 0; c < VC; c++) {
                float f[NT][4];
                #pragma unroll
                for (int i = 0; i < 4; i++) {
                    T y[NT];
                    Terms<T>::split(S[x][c][i], y);
                    #pragma unroll
                    for (int q = 0; q < NT; q++) f[q][i] = ldf(&y[q]);
                }
                #pragma unroll
                for (int q = 0; q < NT; q++)
                    stv<4>(S_s + (q * W + c * 16 + lr) * KS + d0, f[q]);
            }
        }
        lds_barrier();
        load_kv(nx);
        // this wave's 16 queries: the state's part, then the chunk's own
        f32x4 acc[VC] = {}, s[4] = {};
        #pragma unroll
        for (int d = 0; d < DQ; d++) {
            if (d * 32 >= Dp) continue;
            #pragma unroll
            for (int q = 0; q < NT; q++)
                #pragma unroll
                for (int c = 0; c < VC; c++)
                    acc[c] = mma(frag8(S_s + (q * W + c * 16 + lr) * KS
                                       + d * 32 + g * 8), qf[d], acc[c]);
            #pragma unroll
            for (int kt = 0; kt < 4; kt++)
                if (kt <= w)
                    s[kt] = mma(frag8(k_s + (kt * 16 + lr) * KS + d * 32
                                      + g * 8), qf[d], s[kt]);
        }
        load_q(nx);
        #pragma unroll
        for (int c = 0; c < VC; c++) acc[c] *= fade0;
        #pragma unroll
        for (int kt = 0; kt < 4; kt++) s[kt] *= fade[kt];
        #pragma unroll
        for (int hh = 0; hh < 2; hh++) {
            if (hh * 2 > w) continue;
            f32x4 part[NT][2];
            #pragma unroll
            for (int y = 0; y < 2; y++)
                #pragma unroll
                for (int i = 0; i < 4; i++) {
                    T x[NT];
                    Terms<T>::split(s[hh * 2 + y][i], x);
                    #pragma unroll
                    for (int q = 0; q < NT; q++)
                        part[q][y][i] = ldf(&x[q]);
                }
            Frag<T> b[NT];
            #pragma unroll
            for (int q = 0; q < NT; q++) b[q] = weight_frag<T>(part[q]);
            #pragma unroll
            for (int c = 0; c < VC; c++) {
                const Frag<T> v = value_frag(v_s + hh * 32 * VS + c * 16, VS,
                                             lane);
                #pragma unroll
                for (int q = 0; q < NT; q++) acc[c] = mma(v, b[q], acc[c]);
            }
        }
        if (me < n) {
            float* dst = o + ((int64_t)(first + t0 + me) * H + h) * V;
            #pragma unroll
            for (int c = 0; c < VC; c++) {
                const int v = v0 + c * 16 + g * 4;
                if (V % 4 == 0) {
                    if (v < V)
                        *reinterpret_cast<f32x4*>(dst + v) = acc[c];
                } else
                    #pragma unroll
                    for (int i = 0; i < 4; i++)
                        if (v + i < V) dst[v + i] = acc[c][i];
            }
        }
        // the next state
        const float fade_n = pw[n];
        Frag<T> dv[NT][VC][2];
        #pragma unroll
        for (int q = 0; q < NT; q++)
            #pragma unroll
            for (int c = 0; c < VC; c++)
                #pragma unroll
                for (int hh = 0; hh < 2; hh++)
                    dv[q][c][hh] = value_frag(
                        d_s + (q * CH + hh * 32) * VS + c * 16, VS, lane);
        #pragma unroll
        for (int x = 0; x < NS; x++) {
            const int d0 = (w + x * 4) * 16;
            if (d0 >= Dp) continue;
            #pragma unroll
            for (int c = 0; c < VC; c++) S[x][c] *= fade_n;
            #pragma unroll
            for (int hh = 0; hh < 2; hh++) {
                const Frag<T> k = value_frag(k_s + hh * 32 * KS + d0, KS,
                                             lane);
                #pragma unroll
                for (int q = 0; q < NT; q++)
                    #pragma unroll
                    for (int c = 0; c < VC; c++)
                        S[x][c] = mma(k, dv[q][c][hh], S[x][c]);
            }
        }
        lds_barrier();
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

static int lightning_pad(int n, int to) { return (n + to - 1) / to * to; }

// elements of the activation scratch
extern "C" int64_t lightning_scratch(int rows, int H, int D, int V)
{
    return (int64_t)rows * H
           * (2 * lightning_pad(D, 32) + lightning_pad(V, 8));
}

// Portions of whole sequences in chunks of 64 rows.  chunks int32 [n, 2]
// (first row, rows), a sequence's chunks in a run; seqs int32 [m, 2] (first
// chunk, chunks); D <= 256.  Rows row_base .. row_base + rows - 1.
extern "C" int lightning_chunks(
    int f32, void* o, void* scr, const void* p, int p32, int n_part,
    int64_t part_stride, int64_t ld, int oq, int ok, int ov, int act,
    const void* powers, void* state, const void* slot, const void* pos,
    const void* chunks, const void* seqs, int n_seqs, int row_base, int rows,
    int H, int D, int V, hipStream_t stream)
{
    if (D < 1 || V < 1 || D > 256) return (int)hipErrorInvalidValue;
    const int Dp = lightning_pad(D, 32), Vp = lightning_pad(V, 8);
    const bool v8 = D % 8 == 0 && V % 8 == 0 && oq % 8 == 0 && ok % 8 == 0
                    && ov % 8 == 0 && ld % 8 == 0 && part_stride % 8 == 0;
    const int64_t total = (int64_t)rows * H * (2 * Dp + Vp);
    const int64_t want = (total / (v8 ? 8 : 1) + 255) / 256;
    const int ga = (int)(want < 8192 ? want : 8192);
    #define LA_GO(T, P, VE)                                                \
        k_lightning_act<T, P, VE><<<ga, 256, 0, stream>>>(                 \
            (T*)scr, Rows<P>{(const P*)p, n_part, part_stride, ld},        \
            Cols{oq, ok, ov, act}, row_base, rows, total, H, D, V, Dp, Vp)
    #define LA_V(T, P)                                                     \
        do { if (v8) LA_GO(T, P, 8); else LA_GO(T, P, 1); } while (0)
    if (f32) LA_V(float, float);
    else if (p32) LA_V(bf16, float);
    else LA_V(bf16, bf16);
    #undef LA_V
    #undef LA_GO
    // wide strips share the loads of q and k, narrow ones fill the chip
    auto blocks = [&](int vc) {
        return (int64_t)n_seqs * H * ((V + vc * 16 - 1) / (vc * 16));
    };
    const int vc = f32 ? (blocks(2) >= 512 ? 2 : 1)
                   : Dp <= 128 && blocks(4) >= 2048 ? 4
                   : blocks(2) >= 512 ? 2 : 1;
    #define SC(T, NS, VC)                                                  \
        do {                                                               \
            constexpr int es = sizeof(T), pad = 16 / es;                   \
            const int lds = ((CH + Terms<T>::N * VC * 16)                  \
                                 * (NS * 64 + pad)                         \
                             + (1 + Terms<T>::N) * CH * (VC * 16 + pad))   \
                            * es + PW * 4;                                 \
            (void)hipFuncSetAttribute(                                     \
                (const void*)k_lightning_scan<T, NS, VC>,                  \
                hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);   \
            k_lightning_scan<T, NS, VC>                                    \
                <<<dim3(n_seqs, H, (V + VC * 16 - 1) / (VC * 16)), 256,    \
                   lds, stream>>>(                                         \
                    (float*)o, (const T*)scr, (const float*)powers,        \
                    (float*)state, (const int*)slot, (const int*)pos,      \
                    (const int*)chunks, (const int*)seqs, row_base, rows,  \
                    H, D, V, Dp, Vp);                                      \
        } while (0)
    #define SC_NS(T, VC)                                                   \
        do {                                                               \
            if (Dp <= 64) SC(T, 1, VC);                                    \
            else if (Dp <= 128) SC(T, 2, VC);                              \
            else SC(T, 4, VC);                                             \
        } while (0)
    if (f32) { if (vc == 1) SC_NS(float, 1); else SC_NS(float, 2); }
    else if (vc == 4) { if (Dp <= 64) SC(bf16, 1, 4); else SC(bf16, 2, 4); }
    else if (vc == 2) SC_NS(bf16, 2);
    else SC_NS(bf16, 1);
    #undef SC_NS
    #undef SC
    return (int)hipGetLastError();
}
