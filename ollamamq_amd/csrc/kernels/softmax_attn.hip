// gfx950 softmax attention over a paged key/value pool.
//
//   score = scale * q.k over the keys of the query's window
//   out = sum exp(score) v / (sum exp(score) + exp(sink))
//
// The sink, a number per query head, is one more term of the denominator and
// is optional, as is the window.  Instead of a window a query may see its own
// chunk of positions, counted from the sequence's first.  A head's result may
// be gated by the sigmoid of a projected number.  Scores, maxima and sums are
// fp32; in bf16 models exponents are taken in base 2.
//
// All heads of a key/value head are rows of one tile: row = token * R + head
// within the group, R = H / G, so a staged key serves the whole group.
// Pools are [page][G][page_size][width], widths filled up to multiples of 8.
#include "tile_mma.h"

#define NEG (-3.0e38f)

struct Soft {
    float scale;
    const float* sink;                // per query head, or null
    int window, chunk;                // both 0: every earlier key
};
// first key that a query at position p sees
DEV int first_seen(const Soft& rule, int p) {
    if (rule.window > 0) return max(0, p - rule.window + 1);
    return rule.chunk > 0 ? p - p % rule.chunk : 0;
}

// Column `first` + head of a projection, or nothing
struct HeadGate {
    const void* p;
    int f32, n_part;
    int64_t part_stride, ld;
    int first;
};
template <typename T> DEV float gate_of(const HeadGate& q, int64_t t, int h) {
    if (!q.p) return 1.f;
    float z;
    if (sizeof(T) == 4 || q.f32)
        ldrow<1>(Rows<float>{(const float*)q.p, q.n_part, q.part_stride, q.ld},
                 t, q.first + h, &z);
    else
        ldrow<1>(Rows<T>{(const T*)q.p, q.n_part, q.part_stride, q.ld}, t,
                 q.first + h, &z);
    return sigmoid_of<T>(z);
}

// exponentials and the units of a score they take
template <typename T> struct Expo;
template <> struct Expo<float> {
    static constexpr float unit = 1.f;
    static DEV float of(float x) { return expf(x); }
};
template <> struct Expo<bf16> {
    static constexpr float unit = 1.4426950408889634f;
    static DEV float of(float x) { return __builtin_amdgcn_exp2f(x); }
};

// Scores of N tiles of 16 keys become weights; m, l: the row's running
// maximum and sum; the row sees `span` tokens, itself included.  Returns what
// the row's earlier results are scaled by.  A row may have seen no key yet: its weights stay zero.
template <typename T, int N>
DEV float soften(f32x4* s, float c, bool masked, int dist0, int span,
                 float& m, float& l) {
    float mx = NEG;
    #pragma unroll
    for (int j = 0; j < N; j++)
        #pragma unroll
        for (int i = 0; i < 4; i++) {
            float v = s[j][i] * c;
            if (masked) {
                const int d = dist0 - j * 16 - i;
                if (d < 0 || d >= span) v = NEG;
            }
            s[j][i] = v;
            mx = fmaxf(mx, v);
        }
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    const float mn = fmaxf(m, mx);
    const float ref = mn > NEG ? mn : 0.f;
    const float f = Expo<T>::of(m - ref);
    float sum = 0.f;
    #pragma unroll
    for (int j = 0; j < N; j++)
        #pragma unroll
        for (int i = 0; i < 4; i++) {
            const float p = Expo<T>::of(s[j][i] - ref);
            s[j][i] = p;
            sum += p;
        }
    sum += __shfl_xor(sum, 16, 64);
    sum += __shfl_xor(sum, 32, 64);
    l = l * f + sum;
    m = mn;
    return f;
}

// factor of a row's sum of weighted values: maximum m, sum of weights l
template <typename T>
DEV float finish(float m, float l, const float* sink, int h) {
    if (!sink) return 1.f / l;
    const float z = sink[h] * Expo<T>::unit;
    const float top = fmaxf(m, z), e = Expo<T>::of(m - top);
    return e / (l * e + Expo<T>::of(z - top));
}

// ---------------------------------------------------------------------------
// Portions of prompts.  Block: four waves of NQ 16-row tiles over 64-key
// chunks.  S^T = K Q^T puts a row on a lane (16 keys per lane and chunk);
// the weights stay in registers as the operand of the value product.
// Dp <= 32 * DT, Vp <= 16 * VT.
// ---------------------------------------------------------------------------
template <typename T, int DT, int VT, int NQ>
__global__ __launch_bounds__(256, sizeof(T) == 2 && DT <= 4 && VT <= 8
                                       ? 4 - NQ : 1) void k_softmax_flash(
    T* __restrict__ out,               // [T, H, V]
    const T* __restrict__ q,           // [T, H, Dp]
    const T* __restrict__ kpool, const T* __restrict__ vpool,
    const int* __restrict__ ptab, const int* __restrict__ slot,
    const int* __restrict__ pos,
    const int* __restrict__ items,     // [n, 2] first row, rows
    int H, int G, int V, int Dp, int Vp, int pshift, int maxp, Soft rule,
    HeadGate gate)
{
    constexpr int KT = 64;
    constexpr int PAD = 16 / sizeof(T);
    constexpr int KS = DT * 32 + PAD, VS = VT * 16 + PAD;
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    const int lr = lane & 15, g = lane >> 4;
    const int kvh = blockIdx.x, R = H / G;
    const int* it = items + (int64_t)(gridDim.y - 1 - blockIdx.y) * 2;
    const int row0 = it[0], n_rows = it[1];
    const int tok0 = row0 / R, tok1 = (row0 + n_rows - 1) / R;
    const int pos0 = pos[tok0], pos1 = pos[tok1];
    const int* pt = ptab + (int64_t)slot[tok0] * maxp;
    const int kv_len = pos1 + 1;
    const int seen = first_seen(rule, pos0);
    const int last = first_seen(rule, pos1);
    const int c_lo = seen / KT, c_hi = (kv_len + KT - 1) / KT;
    extern __shared__ __attribute__((aligned(16))) char smem[];
    T* k_s = reinterpret_cast<T*>(smem);          // [KT][KS]
    T* v_s = k_s + KT * KS;                       // [KT][VS]

    Frag<T> qf[NQ][DT];
    int qpos[NQ], tok[NQ], head[NQ], span[NQ];
    #pragma unroll
    for (int n = 0; n < NQ; n++) {
        const int f = row0 + min((wid * NQ + n) * 16 + lr, n_rows - 1);
        tok[n] = f / R;
        head[n] = kvh * R + f % R;
        qpos[n] = pos[tok[n]];
        span[n] = qpos[n] - first_seen(rule, qpos[n]) + 1;
        const T* qr = q + ((int64_t)tok[n] * H + head[n]) * Dp;
        #pragma unroll
        for (int d = 0; d < DT; d++) {
            const int c = d * 32 + g * 8;
            qf[n][d] = c < Dp ? frag8(qr + c) : frag_zero<T>();
        }
    }
    const bool live = wid * NQ * 16 < n_rows;     // the wave has rows

    constexpr int NK = DT, NV = VT / 2;           // 8-element pieces a thread
    Frag<T> kp[NK], vp[NV];
    int kpage[NK], vpage[NV];
    const int pmask = (1 << pshift) - 1;
    auto key_at = [&](int base, int k) { return min(base + k, kv_len - 1); };
    auto pages = [&](int base) {
        #pragma unroll
        for (int j = 0; j < NK; j++)
            kpage[j] = pt[key_at(base, (tid + j * 256) / (DT * 4)) >> pshift];
        #pragma unroll
        for (int j = 0; j < NV; j++)
            vpage[j] = pt[key_at(base, (tid + j * 256) / (VT * 2)) >> pshift];
    };
    auto load = [&](int base) {
        #pragma unroll
        for (int j = 0; j < NK; j++) {
            const int u = tid + j * 256;
            const int key = key_at(base, u / (DT * 4));
            const int c = (u % (DT * 4)) * 8;
            const int64_t r = (((int64_t)kpage[j] * G + kvh) << pshift)
                              + (key & pmask);
            kp[j] = c < Dp ? frag8(kpool + r * Dp + c) : frag_zero<T>();
        }
        #pragma unroll
        for (int j = 0; j < NV; j++) {
            const int u = tid + j * 256;
            const int key = key_at(base, u / (VT * 2));
            const int c = (u % (VT * 2)) * 8;
            const int64_t r = (((int64_t)vpage[j] * G + kvh) << pshift)
                              + (key & pmask);
            vp[j] = c < Vp ? frag8(vpool + r * Vp + c) : frag_zero<T>();
        }
    };
    auto store = [&]() {
        #pragma unroll
        for (int j = 0; j < NK; j++) {
            const int u = tid + j * 256;
            *reinterpret_cast<Frag<T>*>(
                k_s + (u / (DT * 4)) * KS + (u % (DT * 4)) * 8) = kp[j];
        }
        #pragma unroll
        for (int j = 0; j < NV; j++) {
            const int u = tid + j * 256;
            *reinterpret_cast<Frag<T>*>(
                v_s + (u / (VT * 2)) * VS + (u % (VT * 2)) * 8) = vp[j];
        }
    };

    const float unit = rule.scale * Expo<T>::unit;
    float m[NQ], l[NQ];
    #pragma unroll
    for (int n = 0; n < NQ; n++) { m[n] = NEG; l[n] = 0.f; }
    f32x4 o[NQ][VT] = {};
    pages(c_lo * KT);
    load(c_lo * KT);
    pages((c_lo + 1) * KT);
    for (int ch = c_lo; ch < c_hi; ++ch) {
        const int base = ch * KT;
        store();
        __syncthreads();
        if (ch + 1 < c_hi) {
            load(base + KT);
            pages(base + 2 * KT);
        }
        if (live) {
            f32x4 s[NQ][4] = {};
            #pragma unroll
            for (int kt = 0; kt < 4; kt++) {
                const T* ar = k_s + (kt * 16 + lr) * KS + g * 8;
                #pragma unroll
                for (int d = 0; d < DT; d++) {
                    const Frag<T> a = frag8(ar + d * 32);
                    #pragma unroll
                    for (int n = 0; n < NQ; n++)
                        s[n][kt] = mma(a, qf[n][d], s[n][kt]);
                }
            }
            const bool inside = base + KT - 1 <= pos0 && base >= last;
            #pragma unroll
            for (int n = 0; n < NQ; n++) {
                const int dist0 = qpos[n] - base - g * 4;
                const float f = soften<T, 4>(s[n], unit, !inside, dist0,
                                             span[n], m[n], l[n]);
                if (!__all(f == 1.f)) {
                    #pragma unroll
                    for (int v = 0; v < VT; v++) o[n][v] *= f;
                }
            }
            #pragma unroll
            for (int h = 0; h < 2; h++) {
                Frag<T> b[NQ];
                #pragma unroll
                for (int n = 0; n < NQ; n++)
                    b[n] = weight_frag<T>(s[n] + h * 2);
                #pragma unroll
                for (int v = 0; v < VT; v++) {
                    const Frag<T> a = value_frag(
                        v_s + h * 32 * VS + v * 16, VS, lane);
                    #pragma unroll
                    for (int n = 0; n < NQ; n++)
                        o[n][v] = mma(a, b[n], o[n][v]);
                }
            }
        }
        __syncthreads();
    }
    #pragma unroll
    for (int n = 0; n < NQ; n++) {
        if ((wid * NQ + n) * 16 + lr >= n_rows) continue;
        const float f = finish<T>(m[n], l[n], rule.sink, head[n])
                        * gate_of<T>(gate, tok[n], head[n]);
        #pragma unroll
        for (int v = 0; v < VT; v++)
            put_out(out, tok[n], head[n], v * 16 + g * 4, H, V, o[n][v] * f,
                    false);
    }
}

// ---------------------------------------------------------------------------
// Decode and short portions: one 16-row tile, every wave on its own 32-key
// steps with its own maximum and sum.  Keys go from memory to the operand
// registers, values through a wave-private LDS tile (they are transposed on
// the way out), both a step ahead; the waves meet once, in the final merge.
// ---------------------------------------------------------------------------
template <typename T, int DT, int VT, int NW>
__global__ __launch_bounds__(NW * 64) void k_softmax_decode(
    T* __restrict__ out,               // [T, H, V] (split == 1)
    float* __restrict__ part,          // [split, T, H, V]
    float* __restrict__ ml,            // [split, T, H, 2] maximum, sum
    const T* __restrict__ q, const T* __restrict__ kpool,
    const T* __restrict__ vpool, const int* __restrict__ ptab,
    const int* __restrict__ slot, const int* __restrict__ pos,
    const int* __restrict__ items,     // null: decode, per_seq a token
    int per_seq, int T_rows, int H, int G, int V, int Dp, int Vp, int pshift,
    int maxp, int split, int frag, Soft rule, HeadGate gate)
{
    constexpr int KT = 32, PAD = 16 / sizeof(T), VS = VT * 16 + PAD;
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    const int lr = lane & 15, g = lane >> 4;
    const int kvh = blockIdx.x, R = H / G;
    int row0, n_rows;
    if (items) {
        row0 = items[blockIdx.y * 2];
        n_rows = items[blockIdx.y * 2 + 1];
    } else {
        const int j = blockIdx.y % per_seq;
        row0 = (blockIdx.y / per_seq) * R + j * 16;
        n_rows = min(16, R - j * 16);
    }
    const int tok0 = row0 / R, tok1 = (row0 + n_rows - 1) / R;
    const int pos0 = pos[tok0], pos1 = pos[tok1];
    const int* pt = ptab + (int64_t)slot[tok0] * maxp;
    const int kv_len = pos1 + 1;
    const int seen = first_seen(rule, pos0);
    const int first = seen / KT;
    const int steps = (kv_len + KT - 1) / KT - first;
    // this wave's steps: every GW-th
    const int GW = split * NW;
    const int gw = blockIdx.z * NW + wid;
    extern __shared__ __attribute__((aligned(16))) char smem[];
    T* v_s = reinterpret_cast<T*>(smem) + wid * KT * VS;

    const int f = row0 + min(lr, n_rows - 1);
    const int tok = f / R, head = kvh * R + f % R;
    const int qpos = pos[tok];
    const int span = qpos - first_seen(rule, qpos) + 1;
    Frag<T> qf[DT], kf[2][DT], vr[VT];
    {
        const T* qr = q + ((int64_t)tok * H + head) * Dp;
        #pragma unroll
        for (int d = 0; d < DT; d++) {
            const int c = d * 32 + g * 8;
            qf[d] = c < Dp ? frag8(qr + c) : frag_zero<T>();
        }
    }
    const int pmask = (1 << pshift) - 1;
    int page[2];
    auto pages = [&](int st) {
        const int base = (first + st) * KT;
        #pragma unroll
        for (int j = 0; j < 2; j++)
            page[j] = pt[min(base + j * 16 + lr, kv_len - 1) >> pshift];
    };
    auto load = [&](int st) {
        const int base = (first + st) * KT;
        #pragma unroll
        for (int j = 0; j < 2; j++) {
            const int key = min(base + j * 16 + lr, kv_len - 1);
            const T* kr = kpool
                + ((((int64_t)page[j] * G + kvh) << pshift)
                   + (key & pmask)) * Dp;
            #pragma unroll
            for (int d = 0; d < DT; d++) {
                const int c = d * 32 + g * 8;
                kf[j][d] = c < Dp ? frag8(kr + c) : frag_zero<T>();
            }
        }
        #pragma unroll
        for (int i = 0; i < VT; i++) {
            const int u = lane + i * 64;
            const int kk = u / (VT * 2), c = (u % (VT * 2)) * 8;
            const int a = __shfl(page[0], kk & 15, 64);
            const int b = __shfl(page[1], kk & 15, 64);
            const int key = min(base + kk, kv_len - 1);
            const int64_t r = (((int64_t)(kk < 16 ? a : b) * G + kvh)
                               << pshift) + (key & pmask);
            vr[i] = c < Vp ? frag8(vpool + r * Vp + c) : frag_zero<T>();
        }
    };
    const float unit = rule.scale * Expo<T>::unit;
    float m = NEG, l = 0.f;
    f32x4 acc[VT] = {};
    if (gw < steps) {
        pages(gw);
        load(gw);
        pages(gw + GW);
    }
    for (int st = gw; st < steps; st += GW) {
        const int base = (first + st) * KT;
        f32x4 s[2] = {};
        #pragma unroll
        for (int d = 0; d < DT; d++) {
            s[0] = mma(kf[0][d], qf[d], s[0]);
            s[1] = mma(kf[1][d], qf[d], s[1]);
        }
        #pragma unroll
        for (int i = 0; i < VT; i++) {
            const int u = lane + i * 64;
            *reinterpret_cast<Frag<T>*>(
                v_s + (u / (VT * 2)) * VS + (u % (VT * 2)) * 8) = vr[i];
        }
        if (st + GW < steps) {
            load(st + GW);
            pages(st + 2 * GW);
        }
        const int dist0 = qpos - base - g * 4;
        const float f = soften<T, 2>(s, unit, true, dist0, span, m, l);
        if (!__all(f == 1.f)) {
            #pragma unroll
            for (int v = 0; v < VT; v++) acc[v] *= f;
        }
        const Frag<T> b = weight_frag<T>(s);
        // the tile is this wave's own: order its writes and reads
        __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
        __builtin_amdgcn_wave_barrier();
        __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
        #pragma unroll
        for (int v = 0; v < VT; v++)
            acc[v] = mma(value_frag(v_s + v * 16, VS, lane), b, acc[v]);
        __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
        __builtin_amdgcn_wave_barrier();
        __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
    }
    __syncthreads();
    f32x4* o_s = reinterpret_cast<f32x4*>(smem);      // [NW][VT][64]
    float* ml_s = reinterpret_cast<float*>(o_s + NW * VT * 64);  // [NW][16][2]
    if (g == 0) {
        ml_s[(wid * 16 + lr) * 2] = m;
        ml_s[(wid * 16 + lr) * 2 + 1] = l;
    }
    __syncthreads();
    float top = NEG, den = 0.f;
    #pragma unroll
    for (int w = 0; w < NW; w++)
        top = fmaxf(top, ml_s[(w * 16 + lr) * 2]);
    #pragma unroll
    for (int w = 0; w < NW; w++)
        den += ml_s[(w * 16 + lr) * 2 + 1]
               * Expo<T>::of(ml_s[(w * 16 + lr) * 2] - top);
    const float mine = Expo<T>::of(m - top);
    #pragma unroll
    for (int v = 0; v < VT; v++)
        o_s[(wid * VT + v) * 64 + lane] = acc[v] * mine;
    __syncthreads();
    if (lr >= n_rows) return;
    const float f0 = split > 1 ? 1.f : finish<T>(top, den, rule.sink, head)
                                       * gate_of<T>(gate, tok, head);
    for (int v = wid; v < VT; v += NW) {
        f32x4 t = o_s[v * 64 + lane];
        #pragma unroll
        for (int w = 1; w < NW; w++) t += o_s[(w * VT + v) * 64 + lane];
        if (split > 1)
            put_out(part + (int64_t)blockIdx.z * T_rows * H * V, tok, head,
                    v * 16 + g * 4, H, V, t, false);
        else put_out(out, tok, head, v * 16 + g * 4, H, V, t * f0, frag);
    }
    if (split > 1 && wid == 0 && g == 0) {
        float* d = ml + (((int64_t)blockIdx.z * T_rows + tok) * H + head) * 2;
        d[0] = top;
        d[1] = den;
    }
}

// merge of the parts' sums for rows t0 .. t0 + n - 1
template <typename T, int VEC>
__global__ __launch_bounds__(256) void k_softmax_combine(
    T* __restrict__ out, const float* __restrict__ part,
    const float* __restrict__ ml, const float* __restrict__ sink,
    HeadGate gate, int t0, int n, int T_rows, int H, int V, int split,
    int frag)
{
    const int N = H * V;
    const int64_t i = ((int64_t)blockIdx.x * 256 + threadIdx.x) * VEC;
    if (i >= (int64_t)n * N) return;
    const int t = t0 + (int)(i / N), c = (int)(i % N), h = c / V;
    const float* d = ml + ((int64_t)t * H + h) * 2;
    const int64_t ds = (int64_t)T_rows * H * 2;
    float top = NEG, den = 0.f;
    for (int s = 0; s < split; s++) top = fmaxf(top, d[s * ds]);
    const float* p = part + (int64_t)t * N + c;
    float v[VEC] = {};
    for (int s = 0; s < split; s++) {
        const float w = Expo<T>::of(d[s * ds] - top);
        den += w * d[s * ds + 1];
        float u[VEC];
        ldv<VEC>(p + (int64_t)s * T_rows * N, u);
        #pragma unroll
        for (int e = 0; e < VEC; e++) v[e] += w * u[e];
    }
    const float f = finish<T>(top, den, sink, h) * gate_of<T>(gate, t, h);
    #pragma unroll
    for (int e = 0; e < VEC; e++) v[e] *= f;
    stv<VEC>(out + (frag ? frag_row_off(t, c, N) : (int64_t)t * N + c), v);
}

template <typename T, int DT, int VT>
static int softmax_go(
    int item_rows, void* out, void* part, void* ml, const void* q,
    const void* kpool,
    const void* vpool, const void* ptab, const void* slot, const void* pos,
    const void* items, int n_items, int per_seq, int T_rows, int H, int G,
    int V, int Dp, int Vp, int pshift, int maxp, int split, int frag,
    Soft rule, HeadGate gate, hipStream_t stream)
{
    constexpr int PAD = 16 / sizeof(T);
    if (item_rows == 16) {
        constexpr int NW = sizeof(T) == 4 || (DT == 8 && VT == 16) ? 4 : 8;
        const int tiles = NW * 32 * (VT * 16 + PAD) * (int)sizeof(T);
        const int sums = NW * VT * 1024 + NW * 128;
        const int lds = tiles > sums ? tiles : sums;
        static bool once = false;
        if (!once) {
            (void)hipFuncSetAttribute(
                (const void*)k_softmax_decode<T, DT, VT, NW>,
                hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
            once = true;
        }
        k_softmax_decode<T, DT, VT, NW>
            <<<dim3(G, n_items, split), NW * 64, lds, stream>>>(
                (T*)out, (float*)part, (float*)ml, (const T*)q,
                (const T*)kpool, (const T*)vpool, (const int*)ptab, (const int*)slot,
                (const int*)pos, (const int*)items, per_seq, T_rows, H, G, V,
                Dp, Vp, pshift, maxp, split, frag, rule, gate);
    } else {
        constexpr int NQ = sizeof(T) == 4 || DT == 8 || VT == 16 ? 1 : 2;
        auto go = item_rows > 64 ? k_softmax_flash<T, DT, VT, NQ>
                                   : k_softmax_flash<T, DT, VT, 1>;
        const int lds = 64 * (DT * 32 + VT * 16 + 2 * PAD) * (int)sizeof(T);
        static bool once = false;
        if (!once) {
            (void)hipFuncSetAttribute(
                (const void*)k_softmax_flash<T, DT, VT, NQ>,
                hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
            (void)hipFuncSetAttribute(
                (const void*)k_softmax_flash<T, DT, VT, 1>,
                hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
            once = true;
        }
        go<<<dim3(G, n_items), 256, lds, stream>>>(
                (T*)out, (const T*)q, (const T*)kpool, (const T*)vpool,
                (const int*)ptab, (const int*)slot, (const int*)pos,
                (const int*)items, H, G, V, Dp, Vp, pshift, maxp, rule,
                gate);
    }
    return (int)hipGetLastError();
}

// most rows of an item of the flash kernel; all of one sequence
extern "C" int softmax_rows(int f32, int Dp, int Vp)
{
    return f32 || Dp > 128 || Vp > 128 ? 64 : 128;
}
// keys a block of the decode kernel takes in one go
extern "C" int softmax_step(int f32) { return f32 ? 128 : 256; }

// item_rows 16: the decode kernel, items null, every token its own sequence,
// or int32 [n, 2] (first row, rows); 64 or 128: the flash kernel.  Tokens
// t0 .. t0 + n_tok - 1 of `out` are written.
extern "C" int softmax_attn(
    int f32, int item_rows, void* out, void* part, void* ml, const void* q,
    const void* kpool, const void* vpool, const void* ptab, const void* slot,
    const void* pos, const void* items, int n_items, int t0, int n_tok,
    int T_rows, int H, int G, int V, int Dp, int Vp, int psz, int maxp,
    int split, int frag, float scale, const void* sink, int window,
    int chunk, const void* gate_p, int g32, int g_parts, int64_t g_stride,
    int64_t g_ld, int og, hipStream_t stream)
{
    if (psz & (psz - 1) || Dp % 8 || Vp % 8 || Dp > 256 || Vp > 256
        || (frag && (f32 || V % 4))
        || (item_rows != 16 && item_rows != 64
            && item_rows != softmax_rows(f32, Dp, Vp)))
        return (int)hipErrorInvalidValue;
    const int pshift = __builtin_ctz(psz);
    const int per_seq = (H / G + 15) / 16;
    Soft rule{scale, (const float*)sink, window, chunk};
    const HeadGate gate{gate_p, g32, g_parts, g_stride, g_ld, og};
    int err;
    #define SA(T, D_, V_)                                                  \
        err = softmax_go<T, D_, V_>(                                       \
            item_rows, out, part, ml, q, kpool, vpool, ptab, slot, pos,    \
            items,                                                         \
            n_items, per_seq, T_rows, H, G, V, Dp, Vp, pshift, maxp,       \
            split, frag, rule, gate, stream)
    #define SA_V(T, D_)                                                    \
        do {                                                               \
            if (Vp <= 64) SA(T, D_, 4);                                    \
            else if (Vp <= 128) SA(T, D_, 8);                              \
            else SA(T, D_, 16);                                            \
        } while (0)
    #define SA_D(T)                                                        \
        do {                                                               \
            if (Dp <= 64) SA_V(T, 2);                                      \
            else if (Dp <= 96) SA_V(T, 3);                                 \
            else if (Dp <= 128) SA_V(T, 4);                                \
            else SA_V(T, 8);                                               \
        } while (0)
    if (f32) SA_D(float); else SA_D(bf16);
    #undef SA_D
    #undef SA_V
    #undef SA
    if (err || item_rows != 16 || split == 1) return err;
    const int N = H * V;
    const int64_t all = (int64_t)n_tok * N;
    #define SC(T, VE)                                                      \
        k_softmax_combine<T, VE>                                           \
            <<<(int)((all / VE + 255) / 256), 256, 0, stream>>>(           \
                (T*)out, (const float*)part, (const float*)ml,             \
                (const float*)sink, gate, t0, n_tok, T_rows, H, V, split, frag)
    if (f32) { if (V % 4) SC(float, 1); else SC(float, 4); }
    else { if (V % 4) SC(bf16, 1); else SC(bf16, 4); }
    #undef SC
    return (int)hipGetLastError();
}
