// gfx950 latent attention: a paged pool caches one row per token, the latent
// c of R values and, if heads have a rotated part, the one rotated key part
// r of Dr values that they share.  Keys and values are linear maps of the
// latent (k = W_uk c, v = W_uv c, per head), the key followed by r.  Two
// exact ways to attend, chosen per sequence by the caller:
//
// * absorbed (decode, short portions): q' = (W_uk^T q, rotated q) makes the
//   score q' . (c, r), so all heads share the cached row — the pool is read
//   once per token of context.  k_latent_attn streams the pool with the
//   (token, head) rows on the matrix cores and returns the weighted latent
//   per row, which k_head_gemm maps through W_uv.
// * expanded (long portions): k and v of the visible context are made with
//   one matrix product each, then k_flash is an ordinary causal flash
//   attention with free key and value widths.
//
// In both a query may see a window of tokens only, itself included, and the
// result may be gated by the sigmoid of a column of the fused projection.
// Cached rows are KW wide, R + Dr filled up with zeros.
#include "tile_mma.h"

#define NEG (-3.0e38f)

// ---------------------------------------------------------------------------
// out[t][h][n] = sum_k x[t*xs + h*hs + k] * w[h][n][k], times the sigmoid of
// a gate column h*N + n.  Rows of `out` are os wide: what follows the N
// columns is copied from behind the row's K inputs (`tail` of them), then
// zeros.
// Grid (n tiles, t / (16*MT), H); a tile is 16 n x 16*MT tokens.  KS == 1:
// a block's four waves make four n tiles; KS == 4: they share one and deal
// its k out (long k, few tiles).  The product is transposed (A = w) so a
// lane stores four consecutive n.
// ---------------------------------------------------------------------------
template <typename T, typename P, int MT, int KS>
__global__ __launch_bounds__(256) void k_head_gemm(
    T* __restrict__ out, const T* __restrict__ x, const T* __restrict__ w,
    Rows<P> gate, int og, int T_rows, int H, int N, int K, int64_t xs,
    int hs, int os, int tail, int frag)
{
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    const int lr = lane & 15, g = lane >> 4;
    const int h = blockIdx.z;
    const int n0 = (KS == 1 ? blockIdx.x * 4 + wid : blockIdx.x) * 16;
    const int t0 = blockIdx.y * 16 * MT;
    if (os > N && blockIdx.x == 0) {
        const int more = os - N;
        for (int i = threadIdx.x; i < 16 * MT * more; i += 256) {
            const int64_t t = t0 + i / more;
            const int j = i % more;
            if (t < T_rows)
                stf(out + (t * H + h) * os + N + j,
                    j < tail ? ldf(x + t * xs + (int64_t)h * hs + K + j)
                             : 0.f);
        }
    }
    if (n0 >= N) return;                    // KS == 4: the whole block
    const T* wr = w + ((int64_t)h * N + min(n0 + lr, N - 1)) * K;
    const T* xr[MT];
    #pragma unroll
    for (int m = 0; m < MT; m++)
        xr[m] = x + (int64_t)min(t0 + m * 16 + lr, T_rows - 1) * xs
                + (int64_t)h * hs;
    f32x4 acc[MT] = {};
    const bool vec = K % 8 == 0 && xs % 8 == 0 && hs % 8 == 0;
    const int k_lo = (KS == 1 ? 0 : wid * 32) + g * 8;
    if (vec) {
        #pragma unroll 4
        for (int k = k_lo; k - g * 8 < K; k += 32 * KS) {
            const Frag<T> a = k < K ? frag8(wr + k) : frag_zero<T>();
            #pragma unroll
            for (int m = 0; m < MT; m++)
                acc[m] = mma(a, k < K ? frag8(xr[m] + k) : frag_zero<T>(),
                             acc[m]);
        }
    } else {
        for (int k = k_lo; k - g * 8 < K; k += 32 * KS) {
            const Frag<T> a = frag_guard(wr, k, K);
            #pragma unroll
            for (int m = 0; m < MT; m++)
                acc[m] = mma(a, frag_guard(xr[m], k, K), acc[m]);
        }
    }
    if constexpr (KS == 4) {
        __shared__ f32x4 red[4][MT][64];
        #pragma unroll
        for (int m = 0; m < MT; m++) red[wid][m][lane] = acc[m];
        __syncthreads();
        if (wid >= MT) return;
        acc[0] = (red[0][wid][lane] + red[1][wid][lane])
                 + (red[2][wid][lane] + red[3][wid][lane]);
    }
    #pragma unroll
    for (int m = 0; m < (KS == 4 ? 1 : MT); m++) {
        const int t = t0 + (KS == 4 ? wid : m) * 16 + lr;
        const int n = n0 + g * 4;
        if (t >= T_rows || n >= N) continue;
        T* o = out + (frag ? frag_row_off(t, h * N + n, H * N)
                           : ((int64_t)t * H + h) * os + n);
        if (gate.p) {
            #pragma unroll
            for (int i = 0; i < 4; i++) {
                float z;
                if (n + i >= N) break;
                ldrow<1>(gate, t, og + h * N + n + i, &z);
                acc[m][i] *= sigmoid_of<T>(z);
            }
        }
        if (N % 4 == 0 && os % 4 == 0) {
            float v[4] = {acc[m][0], acc[m][1], acc[m][2], acc[m][3]};
            stv<4>(o, v);
        } else
            for (int i = 0; i < 4; i++)
                if (n + i < N) stf(o + i, acc[m][i]);
    }
}

// frag: out in the activation-fragment layout (N % 8 == 0); gate may be null
extern "C" int head_gemm(int f32, void* out, const void* x, const void* w,
                         const void* gate, int g32, int n_part,
                         int64_t part_stride, int64_t gate_ld, int og,
                         int T_rows, int H, int N, int K, int64_t xs, int hs,
                         int os, int tail, int frag, hipStream_t stream)
{
    if ((frag && (N % 8 || os != N)) || os < N || tail > os - N)
        return (int)hipErrorInvalidValue;
    const bool wide = T_rows > 16, deal = K >= 256;
    dim3 grid(deal ? (N + 15) / 16 : (N + 63) / 64,
              (T_rows + (wide ? 31 : 15)) / (wide ? 32 : 16), H);
    #define HG_GO(T, P, M, S)                                              \
        k_head_gemm<T, P, M, S><<<grid, 256, 0, stream>>>(                 \
            (T*)out, (const T*)x, (const T*)w,                             \
            Rows<P>{(const P*)gate, n_part, part_stride, gate_ld}, og,     \
            T_rows, H, N, K, xs, hs, os, tail, frag)
    #define HG_K(T, P, M)                                                  \
        do {                                                               \
            if (deal) HG_GO(T, P, M, 4); else HG_GO(T, P, M, 1);           \
        } while (0)
    #define HG_M(T, P)                                                     \
        do { if (wide) HG_K(T, P, 2); else HG_K(T, P, 1); } while (0)
    if (f32) HG_M(float, float);
    else if (g32) HG_M(bf16, float);
    else HG_M(bf16, bf16);
    #undef HG_M
    #undef HG_K
    #undef HG_GO
    return (int)hipGetLastError();
}

// ---------------------------------------------------------------------------
// Absorbed attention over the paged latent pool.
//
// Rows are (token, head) pairs, row = token * H + head; a work item is up to
// M = 16*MT consecutive rows of one sequence, and grid.y cuts its context
// into segments (exact merge in k_latent_combine).  Per KT-key chunk, staged
// once into LDS for all rows:
//   S^T[key, row] = C q'^T      key tiles dealt over the four waves
//   online softmax              16 lanes a row, fp32
//   O^T[r, row]  += C^T P^T     latent columns dealt over the four waves
// NT: 16-wide latent column tiles per wave (R <= 64 * NT).
// ---------------------------------------------------------------------------
template <typename T, int MT, int KT, int NT>
__global__ __launch_bounds__(256) void k_latent_attn(
    T* __restrict__ out,               // [rows, R]      (split == 1)
    T* __restrict__ o_part,            // [split, rows, R]
    float* __restrict__ ml_part,       // [split, rows, 2]
    const T* __restrict__ q,           // [rows, KW]
    const T* __restrict__ pool,        // [pages, psz, KW]
    const int* __restrict__ ptab, const int* __restrict__ slot,
    const int* __restrict__ pos,
    const int* __restrict__ items,     // [n, 2] first row, rows; null: decode
    int per_seq,                       // decode: items per sequence
    int H, int R, int KW, int pshift, int maxp, float scale, int window,
    int64_t rows_total, int split)     // pages of 1 << pshift tokens
{
    constexpr int M = 16 * MT;
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    const int lr = lane & 15, g = lane >> 4;
    int row0, n_rows;
    if (items) {
        row0 = items[blockIdx.x * 2];
        n_rows = items[blockIdx.x * 2 + 1];
    } else {
        const int j = blockIdx.x % per_seq;
        row0 = (blockIdx.x / per_seq) * H + j * M;
        n_rows = min(M, H - j * M);
    }
    const int tok0 = row0 / H, tok1 = (row0 + n_rows - 1) / H;
    const int kv_len = pos[tok1] + 1;
    const int* pt = ptab + (int64_t)slot[tok0] * maxp;
    const int c_first = window > 0 ? max(0, pos[tok0] + 1 - window) / KT : 0;
    const int n_chunks = (kv_len + KT - 1) / KT - c_first;
    const int c_lo = c_first + (int)((int64_t)blockIdx.y * n_chunks / split);
    const int c_hi = c_first
        + (int)((int64_t)(blockIdx.y + 1) * n_chunks / split);

    const int Rp = (KW + 31) & ~31;
    const int cs = Rp + 16 / (int)sizeof(T);      // LDS row strides
    constexpr int SS = KT + 4, PS = KT + 16 / (int)sizeof(T);
    extern __shared__ __attribute__((aligned(16))) char smem[];
    T* q_s = reinterpret_cast<T*>(smem);          // [M][cs]
    T* c_s = q_s + M * cs;                        // [KT][cs]
    T* p_s = c_s + KT * cs;                       // [M][PS]
    float* s_s = reinterpret_cast<float*>(p_s + M * PS);   // [M][SS]
    float* m_s = s_s + M * SS;                    // [M] running max
    float* l_s = m_s + M;                         // [M] running sum
    float* f_s = l_s + M;                         // [M] this chunk's rescale
    int* lim_s = reinterpret_cast<int*>(f_s + M); // [M] visible keys

    const bool vec = KW % 8 == 0;
    // rows of the chunk or of q, zero beyond KW
    auto stage = [&](T* dst, const T* src_row, int c8) {
        const int k = c8 * 8;
        Frag<T> v;
        if (src_row == nullptr) v = frag_zero<T>();
        else if (vec) v = k < KW ? frag8(src_row + k) : frag_zero<T>();
        else v = frag_guard(src_row, k, KW);
        *reinterpret_cast<Frag<T>*>(dst + k) = v;
    };
    const int n8 = Rp / 8;
    for (int u = tid; u < M * n8; u += 256) {
        const int r = u / n8;
        stage(q_s + r * cs,
              r < n_rows ? q + (int64_t)(row0 + r) * KW : nullptr, u % n8);
    }
    if (tid < M) {
        m_s[tid] = NEG;
        l_s[tid] = 0.f;
        lim_s[tid] = tid < n_rows ? pos[(row0 + tid) / H] + 1 : 0;
    }
    // this thread's 8-element pieces of a chunk: (key, column) of each
    constexpr int NP = KT * NT / 32;
    Frag<T> piece[NP];
    int where[NP];
    #pragma unroll
    for (int j = 0; j < NP; j++) {
        const int u = tid + j * 256;
        where[j] = u < KT * n8 ? (u / n8) << 16 | (u % n8) * 8 : -1;
    }
    // Loads are unconditional, with keys and columns clamped to valid ones:
    // a key past the end has weight zero, a column past KW meets zeros of q'
    // or is not stored.  Page numbers are fetched a chunk ahead.
    const int pmask = (1 << pshift) - 1;
    int page[NP];
    auto key_of = [&](int j, int base) {
        return min(base + (max(where[j], 0) >> 16), kv_len - 1);
    };
    auto pages = [&](int base) {
        #pragma unroll
        for (int j = 0; j < NP; j++) page[j] = pt[key_of(j, base) >> pshift];
    };
    auto fetch = [&](int base) {
        #pragma unroll
        for (int j = 0; j < NP; j++) {
            const int c = max(where[j], 0) & 0xffff;
            const T* src = pool + (((int64_t)page[j] << pshift)
                                   + (key_of(j, base) & pmask)) * KW;
            if (vec) piece[j] = frag8(src + min(c, KW - 8));
            else piece[j] = frag_guard(src, c, KW);
        }
    };
    f32x4 acc[MT][NT] = {};
    __syncthreads();               // a segment may hold no chunk at all

    if (c_lo < c_hi) {
        pages(c_lo * KT);
        fetch(c_lo * KT);
        pages((c_lo + 1) * KT);
    }
    for (int ch = c_lo; ch < c_hi; ++ch) {
        const int base = ch * KT;
        #pragma unroll
        for (int j = 0; j < NP; j++)
            if (where[j] >= 0)
                *reinterpret_cast<Frag<T>*>(
                    c_s + (where[j] >> 16) * cs + (where[j] & 0xffff))
                    = piece[j];
        __syncthreads();
        if (ch + 1 < c_hi) {
            fetch(base + KT);
            pages(base + 2 * KT);
        }
        #pragma unroll
        for (int i = 0; i < (MT * KT / 16 + 3) / 4; i++) {
            const int id = wid + i * 4;
            if (id < MT * KT / 16) {
                const int mt = id / (KT / 16), kt = id % (KT / 16);
                f32x4 s = {};
                const T* ar = c_s + (kt * 16 + lr) * cs + g * 8;
                const T* br = q_s + (mt * 16 + lr) * cs + g * 8;
                for (int k = 0; k < Rp; k += 32)
                    s = mma(frag8(ar + k), frag8(br + k), s);
                const int row = mt * 16 + lr, k0 = kt * 16 + g * 4;
                #pragma unroll
                for (int e = 0; e < 4; e++) {
                    const int d = lim_s[row] - (base + k0 + e);
                    s[e] = d > 0 && (window <= 0 || d <= window)
                               ? s[e] * scale : NEG;
                }
                *reinterpret_cast<f32x4*>(s_s + row * SS + k0) = s;
            }
        }
        __syncthreads();
        // 16 lanes a row, KT/16 keys a lane
        #pragma unroll
        for (int mt = 0; mt < MT; mt++) {
            const int row = mt * 16 + wid * 4 + g;
            constexpr int KL = KT / 16;
            float s[KL], mx = NEG;
            #pragma unroll
            for (int j = 0; j < KL; j++) {
                s[j] = s_s[row * SS + lr + j * 16];
                mx = fmaxf(mx, s[j]);
            }
            #pragma unroll
            for (int o = 8; o; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o, 64));
            const float m_old = m_s[row], m_new = fmaxf(m_old, mx);
            float sum = 0.f;
            #pragma unroll
            for (int j = 0; j < KL; j++) {
                const float p = s[j] > NEG ? exp_of<T>(s[j] - m_new) : 0.f;
                sum += p;
                stf(p_s + row * PS + lr + j * 16, p);
            }
            #pragma unroll
            for (int o = 8; o; o >>= 1) sum += __shfl_xor(sum, o, 64);
            if (lr == 0) {
                const float f = exp_of<T>(m_old - m_new);
                f_s[row] = f;
                l_s[row] = l_s[row] * f + sum;
                m_s[row] = m_new;
            }
        }
        __syncthreads();
        float f[MT];
        #pragma unroll
        for (int mt = 0; mt < MT; mt++) f[mt] = f_s[mt * 16 + lr];
        #pragma unroll
        for (int n = 0; n < NT; n++) {
            const int col = (n * 4 + wid) * 16 + lr;
            if ((n * 4 + wid) * 16 < R) {
                #pragma unroll
                for (int mt = 0; mt < MT; mt++) acc[mt][n] *= f[mt];
                #pragma unroll
                for (int k = 0; k < KT; k += 32) {
                    Frag<T> a;
                    #pragma unroll
                    for (int e = 0; e < 8; e++) {
                        const int key = k + g * 8 + e;
                        if constexpr (KT >= 32)
                            frag_set(a, e, ldf(c_s + key * cs + col));
                        else
                            frag_set(a, e, key < KT
                                     ? ldf(c_s + key * cs + col) : 0.f);
                    }
                    #pragma unroll
                    for (int mt = 0; mt < MT; mt++) {
                        const T* br = p_s + (mt * 16 + lr) * PS + k + g * 8;
                        Frag<T> b;
                        if (KT >= 32 || g < 2) b = frag8(br);
                        else b = frag_zero<T>();
                        acc[mt][n] = mma(a, b, acc[mt][n]);
                    }
                }
            }
        }
        __syncthreads();
    }

    #pragma unroll
    for (int mt = 0; mt < MT; mt++) {
        const int row = mt * 16 + lr;
        if (row >= n_rows) continue;
        const int64_t gr = row0 + row;
        const float l = l_s[row];
        const float inv = l > 0.f ? 1.f / l : 0.f;
        #pragma unroll
        for (int n = 0; n < NT; n++) {
            const int c0 = (n * 4 + wid) * 16 + g * 4;
            T* dst = split > 1
                ? o_part + ((int64_t)blockIdx.y * rows_total + gr) * R + c0
                : out + gr * R + c0;
            float v[4];
            #pragma unroll
            for (int i = 0; i < 4; i++) v[i] = acc[mt][n][i] * inv;
            if (R % 4 == 0) {
                if (c0 < R) stv<4>(dst, v);
            } else
                #pragma unroll
                for (int i = 0; i < 4; i++)
                    if (c0 + i < R) stf(dst + i, v[i]);
        }
        if (split > 1 && wid == 0 && g == 0) {
            float* d = ml_part
                + ((int64_t)blockIdx.y * rows_total + gr) * 2;
            d[0] = m_s[row];
            d[1] = l;
        }
    }
}

// ---------------------------------------------------------------------------
// The same for bf16 with KW <= 16 * NT, R <= 16 * NV, KW % 8 == 0 and
// R % 4 == 0: every wave is a whole attention of its own.  Wave (row tile rh, key group kh) holds its q' rows
// as matrix operands and its [R, 16] result in registers and takes its own
// keys of each 64-key chunk:
//   S^T = C q'^T, so a lane holds one row's scores for keys 4g + i, which is
//   the operand layout of the second product: P never leaves the lane;
//   O^T += C^T P^T with C^T read through the LDS transpose load.
// The waves meet only at the double-buffered chunk and in the last merge.
// ---------------------------------------------------------------------------
template <int NT, int NV, int RH>
__global__ __launch_bounds__(256, 1) void k_latent_mq(
    bf16* __restrict__ out, bf16* __restrict__ o_part,
    float* __restrict__ ml_part, const bf16* __restrict__ q,
    const bf16* __restrict__ pool, const int* __restrict__ ptab,
    const int* __restrict__ slot, const int* __restrict__ pos,
    const int* __restrict__ items, int per_seq, int H, int R, int KW,
    int pshift, int maxp, float scale, int window, int64_t rows_total,
    int split)
{
    constexpr int M = 16 * RH, KH = 4 / RH, NK = 4 / KH, KT = 64;
    constexpr int Rp = NT * 16, CS = Rp + 8;
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    const int lr = lane & 15, g = lane >> 4;
    const int rh = wid % RH, kh = wid / RH;
    int row0, n_rows;
    if (items) {
        row0 = items[blockIdx.x * 2];
        n_rows = items[blockIdx.x * 2 + 1];
    } else {
        const int j = blockIdx.x % per_seq;
        row0 = (blockIdx.x / per_seq) * H + j * M;
        n_rows = min(M, H - j * M);
    }
    const int tok0 = row0 / H, tok1 = (row0 + n_rows - 1) / H;
    const int kv_len = pos[tok1] + 1;
    const int* pt = ptab + (int64_t)slot[tok0] * maxp;
    const int c_first = window > 0 ? max(0, pos[tok0] + 1 - window) / KT : 0;
    const int n_chunks = (kv_len + KT - 1) / KT - c_first;
    const int c_lo = c_first + (int)((int64_t)blockIdx.y * n_chunks / split);
    const int c_hi = c_first
        + (int)((int64_t)(blockIdx.y + 1) * n_chunks / split);
    extern __shared__ __attribute__((aligned(16))) char smem[];
    bf16* c_s = reinterpret_cast<bf16*>(smem);    // [2][KT][CS]

    const int row = rh * 16 + lr;
    const int my_lim = row < n_rows ? pos[(row0 + row) / H] + 1 : 0;
    bf16x8 qf[NT / 2];
    {
        const bf16* qr = q + (int64_t)(row0 + min(row, n_rows - 1)) * KW;
        #pragma unroll
        for (int k = 0; k < NT / 2; k++) {
            const int c = k * 32 + g * 8;
            qf[k] = c < KW ? frag8(qr + c) : frag_zero<bf16>();
        }
    }
    // pieces of a chunk, NT*2 in a row: the first MP of every row, a power of
    // two, then the rest.  With 64 of them a wave reads one row, whose page
    // is a scalar.
    constexpr int MP = NT * 2 >= 64 ? 64 : NT * 2 >= 32 ? 32 : 16;
    constexpr int XP = NT * 2 - MP, MJ = KT * MP / 256;
    constexpr int NP = MJ + KT * XP / 256;
    const int wave = __builtin_amdgcn_readfirstlane(wid);
    auto row_of = [&](int j) {
        if (j < MJ) return MP == 64 ? j * 4 + wave : (tid + j * 256) / MP;
        return (tid + (j - MJ) * 256) / (XP ? XP : 1);
    };
    auto col_of = [&](int j) {
        if (j < MJ) return tid % MP * 8;
        return (MP + tid % (XP ? XP : 1)) * 8;
    };
    bf16x8 piece[NP];
    const int pmask = (1 << pshift) - 1;
    int page[NP];
    auto key_of = [&](int j, int base) {
        return min(base + row_of(j), kv_len - 1);
    };
    auto pages = [&](int base) {
        #pragma unroll
        for (int j = 0; j < NP; j++) page[j] = pt[key_of(j, base) >> pshift];
    };
    auto fetch = [&](int base) {
        #pragma unroll
        for (int j = 0; j < NP; j++) {
            const int c = min(col_of(j), KW - 8);
            piece[j] = frag8(pool + (((int64_t)page[j] << pshift)
                                     + (key_of(j, base) & pmask)) * KW + c);
        }
    };
    auto put = [&](int buf) {
        #pragma unroll
        for (int j = 0; j < NP; j++)
            *reinterpret_cast<bf16x8*>(
                c_s + (buf * KT + row_of(j)) * CS + col_of(j)) = piece[j];
    };
    f32x4 acc[NV] = {};
    float m = NEG, l = 0.f;
    if (c_lo < c_hi) {
        pages(c_lo * KT);
        fetch(c_lo * KT);
        pages((c_lo + 1) * KT);
        put(0);
    }
    __syncthreads();
    for (int ch = c_lo; ch < c_hi; ++ch) {
        const int base = ch * KT + kh * NK * 16;
        const bf16* ct = c_s + (((ch - c_lo) & 1) * KT + kh * NK * 16) * CS;
        if (ch + 1 < c_hi) {
            fetch((ch + 1) * KT);
            pages((ch + 2) * KT);
        }
        f32x4 s[NK] = {};
        {
            f32x4 odd[NK] = {};              // two chains per tile
            #pragma unroll
            for (int k = 0; k < NT / 2; k++)
                #pragma unroll
                for (int j = 0; j < NK; j++) {
                    const bf16x8 a = frag8(ct + (j * 16 + lr) * CS + k * 32
                                           + g * 8);
                    if (k & 1) odd[j] = mma(a, qf[k], odd[j]);
                    else s[j] = mma(a, qf[k], s[j]);
                }
            #pragma unroll
            for (int j = 0; j < NK; j++) s[j] += odd[j];
        }
        float mx = NEG;
        #pragma unroll
        for (int j = 0; j < NK; j++)
            #pragma unroll
            for (int i = 0; i < 4; i++) {
                const int d = my_lim - (base + j * 16 + g * 4 + i);
                const float v = d > 0 && (window <= 0 || d <= window)
                                    ? s[j][i] * scale : NEG;
                s[j][i] = v;
                mx = fmaxf(mx, v);
            }
        mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
        mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
        const float mn = fmaxf(m, mx);
        const float f = __expf(m - mn);
        float sum = 0.f;
        #pragma unroll
        for (int j = 0; j < NK; j++)
            #pragma unroll
            for (int i = 0; i < 4; i++) {
                const float p = s[j][i] > NEG ? __expf(s[j][i] - mn) : 0.f;
                s[j][i] = p;
                sum += p;
            }
        sum += __shfl_xor(sum, 16, 64);
        sum += __shfl_xor(sum, 32, 64);
        l = l * f + sum;
        m = mn;
        if (!__all(f == 1.f)) {
            #pragma unroll
            for (int n = 0; n < NV; n++) acc[n] *= f;
        }
        if constexpr (NK == 2) {
            bf16x8 b;
            #pragma unroll
            for (int i = 0; i < 4; i++) {
                b[i] = (__bf16)s[0][i];
                b[i + 4] = (__bf16)s[1][i];
            }
            #pragma unroll
            for (int n = 0; n < NV; n++) {
                const s16x4 a0 = tr_read(ct + n * 16, CS, lane);
                const s16x4 a1 = tr_read(ct + 16 * CS + n * 16, CS, lane);
                const s16x8 a = __builtin_shufflevector(a0, a1, 0, 1, 2, 3,
                                                        4, 5, 6, 7);
                acc[n] = mma(__builtin_bit_cast(bf16x8, a), b, acc[n]);
            }
        } else {
            bf16x4 b4;
            #pragma unroll
            for (int i = 0; i < 4; i++) b4[i] = (__bf16)s[0][i];
            const s16x4 b = __builtin_bit_cast(s16x4, b4);
            #pragma unroll
            for (int n = 0; n < NV; n++)
                acc[n] = __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(
                    tr_read(ct + n * 16, CS, lane), b, acc[n], 0, 0, 0);
        }
        if (ch + 1 < c_hi) put((ch + 1 - c_lo) & 1);
        __syncthreads();
    }
    // merge the key groups: each wave's scaled result, then a share of the
    // column tiles per wave
    float* ml_s = reinterpret_cast<float*>(smem);           // [4][16][2]
    f32x4* o_s = reinterpret_cast<f32x4*>(smem + 512);      // [4][NV][64]
    if (g == 0) {
        ml_s[(wid * 16 + lr) * 2] = m;
        ml_s[(wid * 16 + lr) * 2 + 1] = l;
    }
    __syncthreads();
    float top = NEG, den = 0.f;
    #pragma unroll
    for (int k = 0; k < KH; k++)
        top = fmaxf(top, ml_s[((k * RH + rh) * 16 + lr) * 2]);
    #pragma unroll
    for (int k = 0; k < KH; k++) {
        const float* d = ml_s + ((k * RH + rh) * 16 + lr) * 2;
        den += d[1] * __expf(d[0] - top);
    }
    const float w = den > 0.f ? __expf(m - top) / den : 0.f;
    #pragma unroll
    for (int n = 0; n < NV; n++)
        o_s[(wid * NV + n) * 64 + lane] = acc[n] * w;
    __syncthreads();
    if (row >= n_rows) return;
    const int64_t gr = row0 + row;
    bf16* dst = split > 1
        ? o_part + ((int64_t)blockIdx.y * rows_total + gr) * R
        : out + gr * R;
    #pragma unroll
    for (int n = 0; n < NV / KH; n++) {
        const int t = kh * (NV / KH) + n;
        f32x4 v = o_s[(rh * NV + t) * 64 + lane];
        #pragma unroll
        for (int k = 1; k < KH; k++)
            v += o_s[((k * RH + rh) * NV + t) * 64 + lane];
        const int c0 = t * 16 + g * 4;
        if (c0 < R) {
            float f4[4] = {v[0], v[1], v[2], v[3]};
            stv<4>(dst + c0, f4);
        }
    }
    if (split > 1 && kh == 0 && g == 0) {
        float* d = ml_part + ((int64_t)blockIdx.y * rows_total + gr) * 2;
        d[0] = top;
        d[1] = den;
    }
}

// merge of the segments' normalised results, weights l e^{m - max}
template <typename T, int VEC>
__global__ __launch_bounds__(128) void k_latent_combine(
    T* __restrict__ out, const T* __restrict__ o_part,
    const float* __restrict__ ml, int64_t row_base, int64_t rows_total,
    int R, int split)                   // split <= 64
{
    const int64_t row = row_base + blockIdx.x;
    const int lane = threadIdx.x & 63;
    __shared__ float w_s[64];
    const float* d = ml + (lane * rows_total + row) * 2;
    const float m = lane < split ? d[0] : NEG;
    const float top = wave_max(m);
    const float e = lane < split ? d[1] * exp_of<T>(m - top) : 0.f;
    const float l = wave_sum(e);
    if (threadIdx.x < 64) w_s[lane] = l > 0.f ? e / l : 0.f;
    __syncthreads();
    for (int c = threadIdx.x * VEC; c < R; c += 128 * VEC) {
        float v[VEC] = {};
        #pragma unroll 4
        for (int s = 0; s < split; s++) {
            float u[VEC];
            ldv<VEC>(o_part + (s * rows_total + row) * R + c, u);
            #pragma unroll
            for (int i = 0; i < VEC; i++) v[i] += w_s[s] * u[i];
        }
        stv<VEC>(out + row * R + c, v);
    }
}

static int latent_lds(int M, int KT, int KW, int esz)
{
    const int cs = ((KW + 31) & ~31) + 16 / esz;
    return (M + KT) * cs * esz + M * (KT + 16 / esz) * esz
           + M * (KT + 4) * 4 + 4 * M * 4;
}

template <typename T, int MT, int KT, int NT>
static int latent_go(
    void* out, void* op, void* mp, const void* q, const void* pool,
    const void* ptab, const void* slot, const void* pos, const void* items,
    int n_items, int per_seq, int H, int R, int KW, int pshift, int maxp,
    float scale, int window, int64_t rows_total, int split,
    hipStream_t stream)
{
    const int lds = latent_lds(16 * MT, KT, KW, sizeof(T));
    static bool once = false;
    if (!once) {
        (void)hipFuncSetAttribute(
            (const void*)k_latent_attn<T, MT, KT, NT>,
            hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
        once = true;
    }
    k_latent_attn<T, MT, KT, NT><<<dim3(n_items, split), 256, lds, stream>>>(
        (T*)out, (T*)op, (float*)mp, (const T*)q, (const T*)pool,
        (const int*)ptab, (const int*)slot, (const int*)pos,
        (const int*)items, per_seq, H, R, KW, pshift, maxp, scale, window,
        rows_total, split);
    return (int)hipGetLastError();
}

// key tiles of k_latent_mq, 0 where it does not apply
static int latent_mq_tiles(int f32, int R, int KW)
{
    if (f32 || KW % 8 || R % 4) return 0;
    if (KW <= 128) return 8;
    if (KW <= 256) return 16;
    if (KW <= 288 && R <= 256) return 18;
    if (KW <= 512) return 32;
    return KW <= 576 && R <= 512 ? 36 : 0;
}

// rows of an item: 16 * latent_mt(f32, H, R, KW)
extern "C" int latent_mt(int f32, int H, int R, int KW)
{
    if (H <= 16) return 1;
    if (latent_mq_tiles(f32, R, KW)) return 2;
    return KW <= 512 && latent_lds(32, 32, KW, f32 ? 4 : 2) <= 160 * 1024
               ? 2 : 1;
}

// items: int32 [n_items, 2] (first row, rows <= 16 * latent_mt), each within
// one sequence; null with per_seq = ceil(H / rows) for a decode batch.
// window 0: all earlier keys.
extern "C" int latent_attn(
    int f32, void* out, void* o_part, void* ml_part, const void* q,
    const void* pool, const void* ptab, const void* slot, const void* pos,
    const void* items, int n_items, int per_seq, int H, int R, int KW,
    int psz, int maxp, float scale, int window, int64_t rows_total,
    int64_t row_base, int64_t rows_here, int split, hipStream_t stream)
{
    if (psz & (psz - 1) || split > 64 || R > KW || KW > 1024)
        return (int)hipErrorInvalidValue;
    const int pshift = __builtin_ctz(psz);
    const int esz = f32 ? 4 : 2;
    const int mt = latent_mt(f32, H, R, KW);
    const int budget = 80 * 1024;            // two blocks a CU if possible
    int kt = 64;
    if (latent_lds(16 * mt, 64, KW, esz) > budget) kt = 32;
    if (latent_lds(16 * mt, kt, KW, esz) > 160 * 1024) kt = 16;
    const int nt = latent_mq_tiles(f32, R, KW);
    if (!nt && latent_lds(16 * mt, kt, KW, esz) > 160 * 1024)
        return (int)hipErrorInvalidValue;
    int err = (int)hipErrorInvalidValue;
    if (nt) {
        auto go = [&](auto* kern, int nv) {
            const int tile = 2 * 64 * (nt * 16 + 8) * 2;
            const int merge = 512 + 4 * nv * 1024;
            const int lds = tile > merge ? tile : merge;
            (void)hipFuncSetAttribute(
                (const void*)kern,
                hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
            kern<<<dim3(n_items, split), 256, lds, stream>>>(
                (bf16*)out, (bf16*)o_part, (float*)ml_part, (const bf16*)q,
                (const bf16*)pool, (const int*)ptab, (const int*)slot,
                (const int*)pos, (const int*)items, per_seq, H, R, KW,
                pshift, maxp, scale, window, rows_total, split);
            err = (int)hipGetLastError();
        };
        #define MQ(N, V)                                                   \
            (mt == 2 ? go(k_latent_mq<N, V, 2>, V)                         \
                     : go(k_latent_mq<N, V, 1>, V))
        if (nt == 8) MQ(8, 8);
        else if (nt == 16) MQ(16, 16);
        else if (nt == 18) MQ(18, 16);
        else if (nt == 32) MQ(32, 32);
        else MQ(36, 32);
        #undef MQ
    } else {
    #define LA(T, M, K, N)                                                 \
        err = latent_go<T, M, K, N>(                                       \
            out, o_part, ml_part, q, pool, ptab, slot, pos, items,         \
            n_items, per_seq, H, R, KW, pshift, maxp, scale, window,       \
            rows_total, split, stream)
    #define LA_N(T, M, K)                                                  \
        do {                                                               \
            if (KW <= 128) LA(T, M, K, 2);                                 \
            else if (KW <= 512) LA(T, M, K, 8);                            \
            else LA(T, 1, K, 16);                                          \
        } while (0)
    #define LA_K(T, M)                                                     \
        do {                                                               \
            if (kt == 64) LA_N(T, M, 64);                                  \
            else if (kt == 32) LA_N(T, M, 32);                             \
            else LA_N(T, M, 16);                                           \
        } while (0)
    #define LA_T(T)                                                        \
        do { if (mt == 2) LA_K(T, 2); else LA_K(T, 1); } while (0)
    if (f32) LA_T(float); else LA_T(bf16);
    }
    #undef LA_T
    #undef LA_K
    #undef LA_N
    #undef LA
    if (err || split == 1) return err;
    #define LC_GO(T, V)                                                    \
        k_latent_combine<T, V><<<(int)rows_here, 128, 0, stream>>>(        \
            (T*)out, (const T*)o_part, (const float*)ml_part, row_base,    \
            rows_total, R, split)
    if (f32) { if (R % 4) LC_GO(float, 1); else LC_GO(float, 4); }
    else { if (R % 4) LC_GO(bf16, 1); else LC_GO(bf16, 4); }
    #undef LC_GO
    return (int)hipGetLastError();
}

// ---------------------------------------------------------------------------
// Causal flash attention with free key width (D + Dr <= 32*DT) and value
// width (<= 16*VT), contiguous keys [kv, H, D], a key part [kv, Dr] that all
// heads share, and TRANSPOSED values [H, V, kv] (the caller's matrix product
// writes them that way).
//
// Block: four waves of NQ 16-query tiles.  S^T = K Q^T puts a query on a
// lane, so its softmax state is two scalars after two cross-lane steps; P
// never leaves registers: the PV product may take keys in any order as long
// as both operands agree, so V^T fragments are read in the order in which
// the lanes already hold P.
// ---------------------------------------------------------------------------
template <typename T, int DT, int VT, int NQ>
__global__ __launch_bounds__(256, sizeof(T) == 2 && DT <= 6 && VT <= 8
                                      ? 2 : 1) void k_flash(
    T* __restrict__ out,               // [T, H, V]
    const T* __restrict__ q,           // [T, ..] row stride qs, head h at
                                       // h * (D + Dr)
    const T* __restrict__ k,           // [kv, H*D]
    const T* __restrict__ kr,          // [kv, ..] row stride krs
    const T* __restrict__ vt,          // [H*V, kv_ld]
    Rows<T> gate, int og,              // gate columns og + h*V, or null
    const int* __restrict__ tiles,     // [n, 4] q row, pos, rows, row of
                                       // position 0 in k, kr and vt
    int H, int D, int Dr, int V, int64_t qs, int64_t krs, int64_t kv_ld,
    float scale, int window)
{
    const int DD = D + Dr;
    constexpr int KT = 64;
    constexpr int PAD = 16 / sizeof(T);
    constexpr int KS = DT * 32 + PAD, VS = KT + PAD;
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    const int lr = lane & 15, g = lane >> 4;
    const int h = blockIdx.x;
    const int* tl = tiles + (int64_t)(gridDim.y - 1 - blockIdx.y) * 4;
    const int q0 = tl[0], pos0 = tl[1], rows = tl[2];
    const int64_t kv0 = tl[3];
    extern __shared__ __attribute__((aligned(16))) char smem[];
    T* k_s = reinterpret_cast<T*>(smem);          // [KT][KS]
    T* v_s = k_s + KT * KS;                       // [VT*16][VS]

    const bool vec = D % 8 == 0 && Dr % 8 == 0 && qs % 8 == 0
                     && (!Dr || (krs % 8 == 0 && (uintptr_t)kr % 16 == 0));
    Frag<T> qf[NQ][DT];
    int qpos[NQ];
    #pragma unroll
    for (int n = 0; n < NQ; n++) {
        const int r = (wid * NQ + n) * 16 + lr;
        qpos[n] = pos0 + r;
        const T* qr = q + (int64_t)(q0 + min(r, rows - 1)) * qs
                      + (int64_t)h * DD;
        #pragma unroll
        for (int d = 0; d < DT; d++) {
            const int c = d * 32 + g * 8;
            if (vec) qf[n][d] = c < DD ? frag8(qr + c) : frag_zero<T>();
            else qf[n][d] = frag_guard(qr, c, DD);
        }
    }
    const T* kh = k + kv0 * H * D + (int64_t)h * D;
    const T* krh = kr + kv0 * krs - D;
    const T* vh = vt + (int64_t)h * V * kv_ld + kv0;
    const int kv_len = pos0 + rows;
    const int n_chunks = (kv_len + KT - 1) / KT;
    const int c_first = window > 0 ? max(0, pos0 + 1 - window) / KT : 0;

    constexpr int NK = DT;                        // 8-element pieces a thread
    constexpr int NV = VT / 2;
    Frag<T> kp[NK], vp[NV];
    auto load = [&](int base) {
        #pragma unroll
        for (int j = 0; j < NK; j++) {
            const int u = tid + j * 256;
            const int key = u / (DT * 4), c = (u % (DT * 4)) * 8;
            const T* src = kh + (int64_t)(base + key) * H * D;
            const T* shared = krh + (base + key) * krs;
            if (vec)
                kp[j] = c < D ? frag8(src + c)
                        : c < DD ? frag8(shared + c) : frag_zero<T>();
            else
                #pragma unroll
                for (int e = 0; e < 8; e++)
                    frag_set(kp[j], e, c + e < D ? ldf(src + c + e)
                             : c + e < DD ? ldf(shared + c + e) : 0.f);
        }
        #pragma unroll
        for (int j = 0; j < NV; j++) {
            const int u = tid + j * 256;
            const int v = u >> 3, c = (u & 7) * 8;
            vp[j] = v < V ? frag8(vh + (int64_t)v * kv_ld + base + c)
                          : frag_zero<T>();
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
            *reinterpret_cast<Frag<T>*>(v_s + (u >> 3) * VS + (u & 7) * 8)
                = vp[j];
        }
    };

    float m[NQ], l[NQ];
    f32x4 o[NQ][VT] = {};
    #pragma unroll
    for (int n = 0; n < NQ; n++) { m[n] = NEG; l[n] = 0.f; }

    load(c_first * KT);
    for (int ch = c_first; ch < n_chunks; ++ch) {
        const int base = ch * KT;
        store();
        __syncthreads();
        if (ch + 1 < n_chunks) load(base + KT);
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
        const bool edge = base + KT > pos0 + 1    // some query sees less
            || (window > 0 && base <= kv_len - 1 - window);
        #pragma unroll
        for (int n = 0; n < NQ; n++) {
            float mx = NEG;
            #pragma unroll
            for (int kt = 0; kt < 4; kt++)
                #pragma unroll
                for (int i = 0; i < 4; i++) {
                    float v = s[n][kt][i] * scale;
                    if (edge) {
                        const int d = qpos[n] - (base + kt * 16 + g * 4 + i);
                        if (d < 0 || (window > 0 && d >= window)) v = NEG;
                    }
                    s[n][kt][i] = v;
                    mx = fmaxf(mx, v);
                }
            mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
            mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
            // a query that has seen no key yet: all its weights are zero
            const float mn = fmaxf(m[n], mx);
            const float ref = mn > NEG ? mn : 0.f;
            const float f = exp_of<T>(m[n] - ref);
            float sum = 0.f;
            #pragma unroll
            for (int kt = 0; kt < 4; kt++)
                #pragma unroll
                for (int i = 0; i < 4; i++) {
                    const float p = exp_of<T>(s[n][kt][i] - ref);
                    s[n][kt][i] = p;
                    sum += p;
                }
            sum += __shfl_xor(sum, 16, 64);
            sum += __shfl_xor(sum, 32, 64);
            l[n] = l[n] * f + sum;
            m[n] = mn;
            #pragma unroll
            for (int v = 0; v < VT; v++) o[n][v] *= f;
        }
        #pragma unroll
        for (int kp2 = 0; kp2 < 2; kp2++) {
            Frag<T> b[NQ];
            #pragma unroll
            for (int n = 0; n < NQ; n++)
                #pragma unroll
                for (int e = 0; e < 4; e++) {
                    frag_set(b[n], e, s[n][kp2 * 2][e]);
                    frag_set(b[n], e + 4, s[n][kp2 * 2 + 1][e]);
                }
            #pragma unroll
            for (int v = 0; v < VT; v++) {
                const T* ar = v_s + (v * 16 + lr) * VS + kp2 * 32 + g * 4;
                const Frag<T> a = frag44(ar, ar + 16);
                #pragma unroll
                for (int n = 0; n < NQ; n++) o[n][v] = mma(a, b[n], o[n][v]);
            }
        }
        __syncthreads();
    }
    #pragma unroll
    for (int n = 0; n < NQ; n++) {
        const int r = (wid * NQ + n) * 16 + lr;
        if (r >= rows) continue;
        const float inv = 1.f / l[n];
        T* orow = out + ((int64_t)(q0 + r) * H + h) * V;
        #pragma unroll
        for (int v = 0; v < VT; v++) {
            const int c = v * 16 + g * 4;
            if (gate.p) {
                #pragma unroll
                for (int i = 0; i < 4; i++) {
                    float z;
                    if (c + i >= V) break;
                    ldrow<1>(gate, q0 + r, og + h * V + c + i, &z);
                    o[n][v][i] *= sigmoid_of<T>(z);
                }
            }
            if (V % 4 == 0) {
                if (c < V) {
                    float w[4];
                    #pragma unroll
                    for (int i = 0; i < 4; i++) w[i] = o[n][v][i] * inv;
                    stv<4>(orow + c, w);
                }
            } else
                #pragma unroll
                for (int i = 0; i < 4; i++)
                    if (c + i < V) stf(orow + c + i, o[n][v][i] * inv);
        }
    }
}

template <typename T, int DT, int VT, int NQ>
static int flash_go(void* out, const void* q, const void* k, const void* kr,
                    const void* vt, const void* gate, int64_t gate_ld,
                    int og, const void* tiles, int n_tiles, int H, int D,
                    int Dr, int V, int64_t qs, int64_t krs, int64_t kv_ld,
                    float scale, int window, hipStream_t stream)
{
    const int pad = 16 / sizeof(T);
    const int lds = (64 * (DT * 32 + pad) + VT * 16 * (64 + pad))
                    * (int)sizeof(T);
    static bool once = false;
    if (!once) {
        (void)hipFuncSetAttribute(
            (const void*)k_flash<T, DT, VT, NQ>,
            hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
        once = true;
    }
    k_flash<T, DT, VT, NQ><<<dim3(H, n_tiles), 256, lds, stream>>>(
        (T*)out, (const T*)q, (const T*)k, (const T*)kr, (const T*)vt,
        Rows<T>{(const T*)gate, 1, 0, gate_ld}, og, (const int*)tiles, H, D,
        Dr, V, qs, krs, kv_ld, scale, window);
    return (int)hipGetLastError();
}

// queries per tile; tiles: int32 [n, 4] (first q row, its position, rows, row
// of position 0 in k / kr / vt); these hold every sequence from a multiple of
// 64 positions on, no later than the first key any query sees, padded to
// another; D + Dr, V <= 256; gate may be null
extern "C" int flash_rows(int f32) { return f32 ? 64 : 128; }

extern "C" int flash_attn(
    int f32, void* out, const void* q, const void* k, const void* kr,
    const void* vt, const void* gate, int64_t gate_ld, int og,
    const void* tiles, int n_tiles, int H, int D, int Dr, int V, int64_t qs,
    int64_t krs, int64_t kv_ld, float scale, int window, hipStream_t stream)
{
    if (D + Dr > 256 || V > 256) return (int)hipErrorInvalidValue;
    int err;
    #define FA(T, D_, V_, Q)                                               \
        err = flash_go<T, D_, V_, Q>(                                      \
            out, q, k, kr, vt, gate, gate_ld, og, tiles, n_tiles, H, D,    \
            Dr, V, qs, krs, kv_ld, scale, window, stream)
    #define FA_V(T, D_, Q)                                                 \
        do {                                                               \
            if (V <= 64) FA(T, D_, 4, Q);                                  \
            else if (V <= 128) FA(T, D_, 8, Q);                            \
            else FA(T, D_, 16, Q);                                         \
        } while (0)
    #define FA_D(T, Q)                                                     \
        do {                                                               \
            if (D + Dr <= 64) FA_V(T, 2, Q);                               \
            else if (D + Dr <= 128) FA_V(T, 4, Q);                         \
            else if (D + Dr <= 192) FA_V(T, 6, Q);                         \
            else FA_V(T, 8, Q);                                            \
        } while (0)
    if (f32) FA_D(float, 1); else FA_D(bf16, 2);
    #undef FA_D
    #undef FA_V
    #undef FA
    return err;
}

// Gather of several sequences' latents in groups of 64 positions: groups
// int32 [n, 3] (slot, first position, rows that exist); the rest is zero.
template <typename T>
__global__ __launch_bounds__(256) void k_latent_gather_groups(
    T* __restrict__ out, const T* __restrict__ pool,
    const int* __restrict__ ptab, const int* __restrict__ groups,
    int R, int psz, int maxp)
{
    const int* gp = groups + (int64_t)blockIdx.x * 3;
    const int* row = ptab + (int64_t)gp[0] * maxp;
    const int base = gp[1], have = gp[2];
    const int wid = threadIdx.x >> 6, lane = threadIdx.x & 63;
    for (int j = blockIdx.y * 16 + wid; j < blockIdx.y * 16 + 16; j += 4) {
        T* dst = out + ((int64_t)blockIdx.x * 64 + j) * R;
        if (j >= have) {
            for (int i = lane; i < R; i += 64) stf(dst + i, 0.f);
            continue;
        }
        const int p = base + j;
        const T* src = pool + ((int64_t)row[p / psz] * psz + p % psz) * R;
        if (R % 8 == 0)
            for (int i = lane * 8; i < R; i += 512)
                *reinterpret_cast<Frag<T>*>(dst + i) = frag8(src + i);
        else
            for (int i = lane; i < R; i += 64) dst[i] = src[i];
    }
}

extern "C" int latent_gather(
    int f32, void* out, const void* pool, const void* ptab,
    const void* groups, int n, int R, int psz, int maxp, hipStream_t stream)
{
    if (f32)
        k_latent_gather_groups<float><<<dim3(n, 4), 256, 0, stream>>>(
            (float*)out, (const float*)pool, (const int*)ptab,
            (const int*)groups, R, psz, maxp);
    else
        k_latent_gather_groups<bf16><<<dim3(n, 4), 256, 0, stream>>>(
            (bf16*)out, (const bf16*)pool, (const int*)ptab,
            (const int*)groups, R, psz, maxp);
    return (int)hipGetLastError();
}
