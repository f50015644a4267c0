// gfx950 mixture of experts: router, and the experts' two products
//
//   share = softmax(router h), the `top` largest kept
//   expert(h) = down (silu(gate h) * (up h))
//
// An assignment a = token * top + rank is one (token, expert) pair.  Gate
// and up rows alternate in blocks of 16, so a tile of the first product
// holds matching pairs and applies the activation before it stores.  The
// second product leaves one row per assignment; the next row kernel adds a
// token's rows up with their shares.  Nothing here needs the host to know
// the routing:
//
// * decode (k_moe_stream): one block per expert and 32 weight rows finds the
//   expert's tokens itself and streams the packed weights once, experts
//   nobody chose cost a look at the list;
// * portions (k_moe_plan, k_moe_gemm, k_moe_mm): assignments are grouped by
//   expert into tiles, then a grouped product over the tiles.
#include "route.h"

typedef __attribute__((ext_vector_type(4))) unsigned u32x4;
typedef __attribute__((ext_vector_type(16))) float f32x16;

// ---------------------------------------------------------------------------
// Router.  Logits, softmax and choice in fp32; equal logits go to the lower
// expert.
// ---------------------------------------------------------------------------

// Few tokens: a block each, its waves deal the experts out.
#define ROUTE_WAVES 8
template <typename T, bool FR>              // FR: h in fragment layout
__global__ __launch_bounds__(ROUTE_WAVES * 64) void k_moe_route_row(
    int* __restrict__ chosen, float* __restrict__ share,   // [T, top]
    const T* __restrict__ h, const T* __restrict__ router, // [T,K], [E,K]
    int K, int E, int top)
{
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    const int t = blockIdx.x;
    extern __shared__ float sm[];            // logits
    for (int e = wid; e < E; e += ROUTE_WAVES) {
        const T* w = router + (int64_t)e * K;
        float s = 0.f;
        #pragma unroll 4
        for (int c = lane * 8; c < K; c += 512) {
            float a[8], b[8];
            ldv<8>(w + c, a);
            ldv<8>(h + (FR ? frag_row_off(t, c, K) : (int64_t)t * K + c), b);
            #pragma unroll
            for (int i = 0; i < 8; i++) s += a[i] * b[i];
        }
        s = wave_sum(s);
        if (lane == 0) sm[e] = s;
    }
    __syncthreads();
    if (tid < 16)
        choose(sm, E, top, tid, chosen + (int64_t)t * top,
               share + (int64_t)t * top, true);
}

// Many tokens: 16 a block on the matrix cores, its waves deal K out.
template <typename T, bool VEC>
__global__ __launch_bounds__(ROUTE_WAVES * 64) void k_moe_route(
    int* __restrict__ chosen, float* __restrict__ share,
    const T* __restrict__ h, const T* __restrict__ router,
    int T_rows, int K, int E, int top)
{
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    const int lr = lane & 15, g = lane >> 4;
    const int t0 = blockIdx.x * 16;
    const int EP = (E + 15) / 16 * 16, LS = EP + 1;
    extern __shared__ float sm[];
    float* part = sm;                            // [waves][16][16]
    float* z = sm + ROUTE_WAVES * 256;           // [16][LS]
    const T* hr = h + (int64_t)min(t0 + lr, T_rows - 1) * K;
    for (int e0 = 0; e0 < EP; e0 += 16) {
        const T* wr = router + (int64_t)min(e0 + lr, E - 1) * K;
        f32x4 acc = {};
        constexpr int STEP = ROUTE_WAVES * 32, U = 4;
        int k = wid * 32 + g * 8;
        if constexpr (VEC) {
            // U steps' loads in flight
            for (; k - g * 8 + (U - 1) * STEP + 32 <= K; k += U * STEP) {
                Frag<T> a[U], b[U];
                #pragma unroll
                for (int u = 0; u < U; u++) {
                    a[u] = frag8(wr + k + u * STEP);
                    b[u] = frag8(hr + k + u * STEP);
                }
                #pragma unroll
                for (int u = 0; u < U; u++) acc = mma(a[u], b[u], acc);
            }
        }
        for (; k - g * 8 < K; k += STEP)
            acc = mma(frag_guard(wr, k, K), frag_guard(hr, k, K), acc);
        #pragma unroll
        for (int i = 0; i < 4; i++)
            part[wid * 256 + (g * 4 + i) * 16 + lr] = acc[i];
        __syncthreads();
        if (tid < 256) {
            float s = 0.f;
            #pragma unroll
            for (int w = 0; w < ROUTE_WAVES; w++) s += part[w * 256 + tid];
            z[(tid & 15) * LS + e0 + (tid >> 4)] = s;
        }
        __syncthreads();
    }
    if (tid >= 256) return;
    const int mt = tid >> 4;
    const int64_t at = (int64_t)(t0 + mt) * top;
    choose(z + mt * LS, E, top, tid & 15, chosen + at, share + at,
           t0 + mt < T_rows);
}

extern "C" int moe_route(
    int f32, void* chosen, void* share, const void* h, const void* router,
    int T_rows, int K, int E, int top, int frag, hipStream_t stream)
{
    const int lds = (ROUTE_WAVES * 256 + 16 * ((E + 15) / 16 * 16 + 1)) * 4;
    if (lds > 64 * 1024 || top > E || (frag && (f32 || K % 64)))
        return (int)hipErrorInvalidValue;
    #define ARGS (int*)chosen, (float*)share
    #define IN(T) (const T*)h, (const T*)router
    #define ROW(T, F)                                                      \
        k_moe_route_row<T, F>                                              \
            <<<T_rows, ROUTE_WAVES * 64, E * 4, stream>>>(ARGS, IN(T), K,  \
                                                          E, top)
    #define TILE(T, V)                                                     \
        k_moe_route<T, V>                                                  \
            <<<(T_rows + 15) / 16, ROUTE_WAVES * 64, lds, stream>>>(       \
                ARGS, IN(T), T_rows, K, E, top)
    const bool vec = K % 8 == 0;
    if (frag) ROW(bf16, true);
    else if (vec && T_rows <= 256) {
        if (f32) ROW(float, false); else ROW(bf16, false);
    } else if (f32) { if (vec) TILE(float, true); else TILE(float, false); }
    else if (vec) TILE(bf16, true);
    else TILE(bf16, false);
    #undef TILE
    #undef ROW
    #undef IN
    #undef ARGS
    return (int)hipGetLastError();
}

// ---------------------------------------------------------------------------
// Group A assignments by expert into tiles of TM.  tile_e[max_tiles]: the
// tile's expert or -1; perm[max_tiles * TM]: the tile's assignments, -1
// fills up.  max_tiles >= A / TM + min(A, E) covers every routing.
// ---------------------------------------------------------------------------
__global__ __launch_bounds__(1024) void k_moe_plan(
    int* __restrict__ tile_e, int* __restrict__ perm,
    const int* __restrict__ chosen, int A, int E, int TM, int max_tiles)
{
    __shared__ int cnt[1024], cur[1024], wsum[16];
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    cnt[tid] = 0;
    __syncthreads();
    constexpr int U = 8;                        // loads in flight
    auto each = [&](auto f) {
        for (int a0 = tid; a0 < A; a0 += 1024 * U) {
            int e[U];
            #pragma unroll
            for (int u = 0; u < U; u++)
                e[u] = chosen[min(a0 + u * 1024, A - 1)];
            #pragma unroll
            for (int u = 0; u < U; u++)
                if (a0 + u * 1024 < A) f(a0 + u * 1024, e[u]);
        }
    };
    each([&](int, int e) { atomicAdd(&cnt[e], 1); });
    __syncthreads();
    const int n = cnt[tid];
    const int tiles = (n + TM - 1) / TM;
    int s = tiles;                              // inclusive scan
    #pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
        const int u = __shfl_up(s, o, 64);
        if (lane >= o) s += u;
    }
    if (lane == 63) wsum[wid] = s;
    __syncthreads();
    int before = 0, total = 0;
    #pragma unroll
    for (int w = 0; w < 16; w++) {
        if (w < wid) before += wsum[w];
        total += wsum[w];
    }
    const int first = before + s - tiles;
    cur[tid] = first * TM;
    for (int m = 0; m < tiles; m++) tile_e[first + m] = tid;
    for (int m = total + tid; m < max_tiles; m += 1024) tile_e[m] = -1;
    __syncthreads();
    for (int e = wid; e < E; e += 16) {         // fill up, a wave an expert
        const int end = (cnt[e] + TM - 1) / TM * TM, p = cur[e];
        for (int i = cnt[e] + lane; i < end; i += 64) perm[p + i] = -1;
    }
    __syncthreads();
    each([&](int a, int e) { perm[atomicAdd(&cur[e], 1)] = a; });
}

extern "C" int moe_plan(
    void* tile_e, void* perm, const void* chosen, int A, int E, int TM,
    int max_tiles, hipStream_t stream)
{
    if (E > 1024 || max_tiles < A / TM + (A < E ? A : E))
        return (int)hipErrorInvalidValue;
    k_moe_plan<<<1, 1024, 0, stream>>>((int*)tile_e, (int*)perm,
                                       (const int*)chosen, A, E, TM,
                                       max_tiles);
    return (int)hipGetLastError();
}

// ---------------------------------------------------------------------------
// Grouped product, any sizes, both types: tiles of 16 assignments, a wave
// per 16 output columns.  GU: out[tile row] = silu(gate) * up, N = 2F weight
// rows; else out[assignment] = W row.  x rows are tokens (GU) or tile rows.
// ---------------------------------------------------------------------------
template <typename T, bool GU, bool VEC>
__global__ __launch_bounds__(256) void k_moe_mm(
    T* __restrict__ out, const T* __restrict__ x, const T* __restrict__ w,
    const int* __restrict__ tile_e, const int* __restrict__ perm, int top,
    int N, int K)
{
    constexpr int NB = GU ? 2 : 1;
    const int e = tile_e[blockIdx.y];
    if (e < 0) return;
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    const int lr = lane & 15, g = lane >> 4;
    const int n0 = (blockIdx.x * 4 + wid) * 16 * NB;
    if (n0 >= N) return;
    const int p = blockIdx.y * 16 + lr;
    const int a = perm[p];
    const T* xr = x + (int64_t)(GU ? max(a, 0) / top : p) * K;
    const T* wr[NB];
    #pragma unroll
    for (int b = 0; b < NB; b++)
        wr[b] = w + ((int64_t)e * N + min(n0 + b * 16 + lr, N - 1)) * K;
    f32x4 acc[NB] = {};
    for (int k = 0; k < K; k += 32) {
        const int c = k + g * 8;
        Frag<T> f;
        if constexpr (VEC) f = c < K ? frag8(xr + c) : frag_zero<T>();
        else f = frag_guard(xr, c, K);
        #pragma unroll
        for (int b = 0; b < NB; b++) {
            Frag<T> m;
            if constexpr (VEC)
                m = c < K ? frag8(wr[b] + c) : frag_zero<T>();
            else m = frag_guard(wr[b], c, K);
            acc[b] = mma(m, f, acc[b]);
        }
    }
    if (GU) {
        const int F = N / 2, f0 = n0 / 2 + g * 4;
        #pragma unroll
        for (int i = 0; i < 4; i++)
            stf(out + (int64_t)p * F + f0 + i,
                silu_of<T>(acc[0][i]) * acc[NB - 1][i]);
    } else if (a >= 0) {
        #pragma unroll
        for (int i = 0; i < 4; i++)
            if (n0 + g * 4 + i < N)
                stf(out + (int64_t)a * N + n0 + g * 4 + i, acc[0][i]);
    }
}

extern "C" int moe_mm(
    int f32, int gu, void* out, const void* x, const void* w,
    const void* tile_e, const void* perm, int n_tiles, int top, int N, int K,
    hipStream_t stream)
{
    if (gu && N % 32) return (int)hipErrorInvalidValue;
    const dim3 grid((N + (gu ? 127 : 63)) / (gu ? 128 : 64), n_tiles);
    #define MM(T, G, V)                                                    \
        k_moe_mm<T, G, V><<<grid, 256, 0, stream>>>(                       \
            (T*)out, (const T*)x, (const T*)w, (const int*)tile_e,         \
            (const int*)perm, top, N, K)
    #define MM_G(T)                                                        \
        do {                                                               \
            if (K % 8) { if (gu) MM(T, true, false);                       \
                         else MM(T, false, false); }                       \
            else { if (gu) MM(T, true, true); else MM(T, false, true); }   \
        } while (0)
    if (f32) MM_G(float); else MM_G(bf16);
    #undef MM_G
    #undef MM
    return (int)hipGetLastError();
}

// ---------------------------------------------------------------------------
// Grouped product for long portions, bf16, K % 64 == 0: 128 x 128 tiles, 64
// deep, four waves of 64 x 64.  Both operands go to LDS by direct loads,
// double buffered; a row is 128 bytes whose eight 16-byte pieces are
// permuted by the row number (the direct load fixes where a lane's piece
// lands, not what it reads), so operand reads spread over the banks.  A
// stage's operands are read to registers before the next stage's loads are
// issued: those then run under the stage's matrix instructions.
// ---------------------------------------------------------------------------
DEV void load_lds16(const bf16* src, bf16* dst) {
    __builtin_amdgcn_global_load_lds(
        (const __attribute__((address_space(1))) void*)src,
        (__attribute__((address_space(3))) void*)dst, 16, 0, 0);
}

template <bool GU>
__global__ __launch_bounds__(256, 2) void k_moe_gemm(
    bf16* __restrict__ out, const bf16* __restrict__ x,
    const bf16* __restrict__ w, const int* __restrict__ tile_e,
    const int* __restrict__ perm, int n_tiles, int top, int N, int K)
{
    constexpr int TM = 128, TN = 128, KT = 64;
    // blocks go round the eight dies: a die takes a run of consecutive
    // tiles, groups of eight row tiles by all column tiles, so that what it
    // works on at a time shares rows and columns in its cache
    const int nt = (N + TN - 1) / TN, total = nt * n_tiles;
    const int id = (blockIdx.x & 7) * (gridDim.x >> 3) + (blockIdx.x >> 3);
    if (id >= total) return;
    const int m8 = id / (8 * nt) * 8, at = id % (8 * nt);
    const int rows8 = min(8, n_tiles - m8);
    const int mt = m8 + at % rows8;
    const int e = tile_e[mt];
    if (e < 0) return;
    __shared__ __attribute__((aligned(16))) bf16 w_s[2][TN * KT];
    __shared__ __attribute__((aligned(16))) bf16 x_s[2][TM * KT];
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    const int lr = lane & 15, g = lane >> 4;
    const int n0 = at / rows8 * TN, p0 = mt * TM;
    // a wave loads 32 rows of each operand, 8 rows an instruction
    const int piece = ((lane & 7) ^ (lane >> 3)) * 8;
    const bf16 *wr[4], *xr[4];
    #pragma unroll
    for (int j = 0; j < 4; j++) {
        const int r = (wid * 4 + j) * 8 + (lane >> 3);
        wr[j] = w + ((int64_t)e * N + min(n0 + r, N - 1)) * K + piece;
        const int64_t row = GU ? max(perm[p0 + r], 0) / top : p0 + r;
        xr[j] = x + row * K + piece;
    }
    auto issue = [&](int buf, int k) {
        #pragma unroll
        for (int j = 0; j < 4; j++) {
            load_lds16(wr[j] + k, w_s[buf] + (wid * 4 + j) * 8 * KT);
            load_lds16(xr[j] + k, x_s[buf] + (wid * 4 + j) * 8 * KT);
        }
    };
    const int wn = wid & 1, wm = wid >> 1;
    f32x4 acc[4][4] = {};
    issue(0, 0);
    for (int k = 0, buf = 0; k < K; k += KT, buf ^= 1) {
        // this wave's loads are done, then everybody's
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __syncthreads();
        bf16x8 a[2][4], b[2][4];
        #pragma unroll
        for (int kk = 0; kk < 2; kk++)
            #pragma unroll
            for (int j = 0; j < 4; j++) {
                const int c = ((kk * 4 + g) ^ (lr & 7)) * 8;
                a[kk][j] = frag8(w_s[buf] + (wn * 64 + j * 16 + lr) * KT + c);
                b[kk][j] = frag8(x_s[buf] + (wm * 64 + j * 16 + lr) * KT + c);
            }
        if (k + KT < K) issue(buf ^ 1, k + KT);
        #pragma unroll
        for (int kk = 0; kk < 2; kk++)
            #pragma unroll
            for (int i = 0; i < 4; i++)
                #pragma unroll
                for (int j = 0; j < 4; j++)
                    acc[i][j] = mma(a[kk][i], b[kk][j], acc[i][j]);
    }
    #pragma unroll
    for (int j = 0; j < 4; j++) {
        const int p = p0 + wm * 64 + j * 16 + lr;
        if (GU) {
            const int F = N / 2;
            #pragma unroll
            for (int i = 0; i < 4; i += 2) {
                const int n = n0 + wn * 64 + i * 16;
                if (n >= N) continue;
                float v[4];
                #pragma unroll
                for (int r = 0; r < 4; r++)
                    v[r] = silu_of<bf16>(acc[i][j][r]) * acc[i + 1][j][r];
                stv<4>(out + (int64_t)p * F + n / 2 + g * 4, v);
            }
        } else {
            const int a = perm[p];
            if (a < 0) continue;
            #pragma unroll
            for (int i = 0; i < 4; i++) {
                const int n = n0 + wn * 64 + i * 16 + g * 4;
                if (n >= N) continue;
                float v[4] = {acc[i][j][0], acc[i][j][1], acc[i][j][2],
                              acc[i][j][3]};
                stv<4>(out + (int64_t)a * N + n, v);
            }
        }
    }
}

extern "C" int moe_gemm(
    int gu, void* out, const void* x, const void* w, const void* tile_e,
    const void* perm, int n_tiles, int top, int N, int K, hipStream_t stream)
{
    if (K % 64 || N % (gu ? 32 : 4)) return (int)hipErrorInvalidValue;
    auto go = gu ? k_moe_gemm<true> : k_moe_gemm<false>;
    const int total = (N + 127) / 128 * n_tiles;
    go<<<(total + 7) / 8 * 8, 256, 0, stream>>>(
        (bf16*)out, (const bf16*)x, (const bf16*)w, (const int*)tile_e,
        (const int*)perm, n_tiles, top, N, K);
    return (int)hipGetLastError();
}

// ---------------------------------------------------------------------------
// The same with packed weights, which need no LDS: a wave reads the matrix
// operands of its own 64 weight rows straight from memory, linearly, 32 deep
// and a step ahead, and multiplies them with all 128 rows of x.  x goes
// through registers to a double-buffered LDS tile, 64 deep, two stages
// ahead, pieces permuted by half the row number (lanes are rows here, and
// of the 16 served together no two share parity and that).  One barrier a stage, which waits for LDS
// only: loads stay in flight across it.
// ---------------------------------------------------------------------------
template <bool GU>
__global__ __launch_bounds__(256, 2) void k_moe_gemm_packed(
    bf16* __restrict__ out, const bf16* __restrict__ x,
    const u32x4* __restrict__ wp, const int* __restrict__ tile_e,
    const int* __restrict__ perm, int n_tiles, int top, int N, int K)
{
    constexpr int TM = 128, TN = 256, KT = 64, NX = 4;
    const int nt = (N + TN - 1) / TN, total = nt * n_tiles;
    const int id = (blockIdx.x & 7) * (gridDim.x >> 3) + (blockIdx.x >> 3);
    if (id >= total) return;
    const int m8 = id / (8 * nt) * 8, at = id % (8 * nt);
    const int rows8 = min(8, n_tiles - m8);
    const int mt = m8 + at % rows8;
    const int e = tile_e[mt];
    if (e < 0) return;
    __shared__ __attribute__((aligned(16))) bf16 x_s[2][TM * KT];
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    const int m = lane & 31, half = lane >> 5;
    const int p0 = mt * TM, n0 = at / rows8 * TN + wid * 64;
    const int tiles = N >> 5, NS = K / KT;
    const bf16x8* wr[2];
    #pragma unroll
    for (int i = 0; i < 2; i++) {
        const int t = min((n0 >> 5) + i, tiles - 1);
        wr[i] = reinterpret_cast<const bf16x8*>(wp)
                + ((int64_t)e * tiles + t) * (K >> 4) * 64 + lane;
    }
    const bf16* xr[NX];
    #pragma unroll
    for (int j = 0; j < NX; j++) {
        const int r = (tid >> 3) + j * 32;
        const int64_t row = GU ? max(perm[p0 + r], 0) / top : p0 + r;
        xr[j] = x + row * K + (tid & 7) * 8;
    }
    bf16* xw = x_s[0] + (tid >> 3) * KT + ((tid & 7) ^ ((tid >> 4) & 7)) * 8;
    bf16x8 xv[NX], w[2][2][2];                 // w[half stage][k step][tile]
    auto load_x = [&](int s) {
        #pragma unroll
        for (int j = 0; j < NX; j++) xv[j] = frag8(xr[j] + s * KT);
    };
    auto store_x = [&](int buf) {
        #pragma unroll
        for (int j = 0; j < NX; j++)
            *reinterpret_cast<bf16x8*>(xw + (buf * TM + j * 32) * KT) = xv[j];
    };
    auto load_w = [&](int b, int h) {          // h: 32-deep step
        #pragma unroll
        for (int kk = 0; kk < 2; kk++)
            #pragma unroll
            for (int i = 0; i < 2; i++)
                w[b][kk][i] = wr[i][(int64_t)(h * 2 + kk) * 64];
    };
    f32x16 acc[2][4] = {};
    load_x(0);
    load_w(0, 0);
    store_x(0);
    if (NS > 1) load_x(1);
    lds_barrier();
    const bf16* xl = x_s[0] + m * KT;
    for (int s = 0; s < NS; s++) {
        const int buf = s & 1;
        #pragma unroll
        for (int b = 0; b < 2; b++) {
            load_w(b ^ 1, min(s * 2 + b + 1, NS * 2 - 1));
            if (b == 0) {
                if (s + 1 < NS) store_x(buf ^ 1);
                if (s + 2 < NS) load_x(s + 2);
            }
            #pragma unroll
            for (int kk = 0; kk < 2; kk++) {
                bf16x8 f[4];
                #pragma unroll
                for (int j = 0; j < 4; j++)
                    f[j] = frag8(xl + (buf * TM + j * 32) * KT
                                 + ((b * 4 + kk * 2 + half) ^ (m >> 1 & 7))
                                       * 8);
                #pragma unroll
                for (int i = 0; i < 2; i++)
                    #pragma unroll
                    for (int j = 0; j < 4; j++)
                        acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(
                            w[b][kk][i], f[j], acc[i][j], 0, 0, 0);
            }
        }
        lds_barrier();
    }
    // a lane holds row m of x and weight rows 8 (r / 4) + 4 half + r % 4
    #pragma unroll
    for (int j = 0; j < 4; j++) {
        const int p = p0 + j * 32 + m;
        const int a = GU ? 0 : perm[p];
        if (a < 0) continue;
        #pragma unroll
        for (int i = 0; i < 2; i++) {
            const int n = n0 + i * 32;
            if (n >= N) continue;
            #pragma unroll
            for (int q = 0; q < (GU ? 2 : 4); q++) {
                float v[4];
                #pragma unroll
                for (int r = 0; r < 4; r++)
                    v[r] = GU ? silu_of<bf16>(acc[i][j][q * 4 + r])
                                    * acc[i][j][(q * 4 + r + 8) & 15]
                              : acc[i][j][q * 4 + r];
                const int c = q * 8 + half * 4;
                stv<4>(GU ? out + (int64_t)p * (N / 2) + n / 2 + c
                          : out + (int64_t)a * N + n + c, v);
            }
        }
    }
}

extern "C" int moe_gemm_packed(
    int gu, void* out, const void* x, const void* wp, const void* tile_e,
    const void* perm, int n_tiles, int top, int N, int K, hipStream_t stream)
{
    if (K % 64 || N % 32) return (int)hipErrorInvalidValue;
    auto go = gu ? k_moe_gemm_packed<true> : k_moe_gemm_packed<false>;
    const int total = (N + 255) / 256 * n_tiles;
    go<<<(total + 7) / 8 * 8, 256, 0, stream>>>(
        (bf16*)out, (const bf16*)x, (const u32x4*)wp, (const int*)tile_e,
        (const int*)perm, n_tiles, top, N, K);
    return (int)hipGetLastError();
}

// ---------------------------------------------------------------------------
// Decode, up to 64 tokens, bf16: block (32 weight rows, expert).  Weights
// are the packed matrix-operand order of the weight-streaming product, x and
// the activation are in fragment layout (x by token, the activation by
// assignment).  The waves deal K out and meet in one sum.
// ---------------------------------------------------------------------------
template <bool GU, int NW>
__global__ __launch_bounds__(NW * 64) void k_moe_stream(
    bf16* __restrict__ act,              // GU: [A, N / 2], fragment layout
    float* __restrict__ out,             // else [A, N]
    const bf16* __restrict__ x, const u32x4* __restrict__ wp,
    const int* __restrict__ chosen, int A, int top, int N, int K)
{
    const int tile = blockIdx.x, e = blockIdx.y;
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
    __shared__ int list[64], count;
    __shared__ float red[NW][32][32];
    if (wid == 0) {
        int n = 0;
        for (int a0 = 0; a0 < A; a0 += 64) {
            const bool mine = a0 + lane < A && chosen[a0 + lane] == e;
            const uint64_t m = __ballot(mine);
            const int at = n + __popcll(m & ((1ull << lane) - 1));
            if (mine && at < 64) list[at] = a0 + lane;
            n += __popcll(m);
        }
        if (lane == 0) count = min(n, 64);
    }
    __syncthreads();
    const int n = count;
    const int NB = K >> 6;
    const int lo = wid * NB / NW, hi = (wid + 1) * NB / NW;
    const u32x4* wb = wp + ((int64_t)e * (N >> 5) + tile) * NB * 256 + lane;
    for (int m0 = 0; m0 < n; m0 += 32) {
        const int a = list[min(m0 + (lane & 31), n - 1)];
        const int src = GU ? a / top : a;
        const bf16x8* xb = reinterpret_cast<const bf16x8*>(x)
            + (int64_t)(src >> 5) * 4 * K + (lane & 32) + (src & 31);
        f32x16 acc = {};
        if (lo < hi) {
            u32x4 b[4];
            bf16x8 f[4];
            auto load = [&](int k) {
                #pragma unroll
                for (int j = 0; j < 4; j++)
                    b[j] = __builtin_nontemporal_load(
                        wb + (int64_t)k * 256 + j * 64);
                #pragma unroll
                for (int j = 0; j < 4; j++)
                    f[j] = xb[(int64_t)k * 256 + j * 64];
            };
            load(lo);
            for (int k = lo; k < hi; k++) {
                #pragma unroll
                for (int j = 0; j < 4; j++)
                    acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(
                        f[j], __builtin_bit_cast(bf16x8, b[j]), acc, 0, 0, 0);
                if (k + 1 < hi) load(k + 1);
            }
        }
        if (m0) __syncthreads();
        #pragma unroll
        for (int r = 0; r < 16; r++)
            red[wid][(r & 3) + 8 * (r >> 2) + 4 * (lane >> 5)][lane & 31]
                = acc[r];
        __syncthreads();
        const int rows = min(32, n - m0);
        constexpr int C = GU ? 16 : 32;
        for (int i = tid; i < rows * C; i += NW * 64) {
            const int m = i / C, c = i % C;
            const int at = list[m0 + m];
            float v = 0.f, u = 0.f;
            #pragma unroll
            for (int s = 0; s < NW; s++) {
                v += red[s][m][c];
                if (GU) u += red[s][m][c + 16];
            }
            if (GU)
                stf(act + frag_row_off(at, tile * 16 + c, N / 2),
                    silu_of<bf16>(v) * u);
            else out[(int64_t)at * N + tile * 32 + c] = v;
        }
    }
}

extern "C" int moe_stream(
    int gu, void* act, void* out, const void* x, const void* wp,
    const void* chosen, int A, int top, int E, int N, int K,
    hipStream_t stream)
{
    if (A / top > 64 || N % 32 || K % 64) return (int)hipErrorInvalidValue;
    const dim3 grid(N / 32, E);
    #define MS(G, W)                                                       \
        k_moe_stream<G, W><<<grid, W * 64, 0, stream>>>(                   \
            (bf16*)act, (float*)out, (const bf16*)x, (const u32x4*)wp,     \
            (const int*)chosen, A, top, N, K)
    if (K >= 2048) { if (gu) MS(true, 8); else MS(false, 8); }
    else { if (gu) MS(true, 4); else MS(false, 4); }
    #undef MS
    return (int)hipGetLastError();
}
