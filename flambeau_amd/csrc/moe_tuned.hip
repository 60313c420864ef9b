// The experts' products on the matrix cores (bfloat16), and a product with few output features.
#include "common.h"
#include "api.h"
#include "recordable.h"

// out[p][:] = scale[p] * (x[src[p]] W_e^T) over the row tiles of fl_moe_route, with v_mfma_f32_16x16x32_bf16.  Every
// expert's matrix is packed as the other products' (a tile of 16 features x 32 k is 1 KB in lane order).
//
// With a gate the matrix holds gate and up rows interleaved in fours, so that gate and up of a feature leave a block in
// lanes 16 apart, and the block stores the activation (bfloat16) in place of both.
#define MG_NONE 0
#define MG_SILU 1
#define MG_CLAMPED 2
typedef GateConstants MoeGate;
template <int GATE>
__device__ __forceinline__ float moe_gate(const MoeGate& m, float g, float u) {
    if constexpr (GATE == MG_CLAMPED) return clamped_gate(g, u, m.alpha, m.limit, m.shift);
    return gate_activation<FL_GATE_SILU>(g) * u;
}
// four values of one place (features f .. f + 3 of the matrix): stored as they are, or with a gate the even quarter
// waves' gates meet the odd ones' ups.  All lanes of a place's column take part.
template <int GATE>
__device__ __forceinline__ void moe_store(const MoeGate& m, void* out, int place, int f, int g, f32x4 v, int N) {
    if constexpr (GATE == MG_NONE) {
        if (f < N) *(f32x4*)((float*)out + (size_t)place * N + f) = v;
    } else {
        f32x4 up;
#pragma unroll
        for (int r = 0; r < 4; ++r) up[r] = __shfl_down(v[r], 16, FL_WAVE);
        if ((g & 1) == 0 && f < N) {
            const bf16x4 o = {(bf16_t)moe_gate<GATE>(m, v[0], up[0]), (bf16_t)moe_gate<GATE>(m, v[1], up[1]),
                              (bf16_t)moe_gate<GATE>(m, v[2], up[2]), (bf16_t)moe_gate<GATE>(m, v[3], up[3])};
            // rows f .. f + 3 (gates) and f + 4 .. f + 7 (ups) of the matrix are features f / 2 .. f / 2 + 3
            *(bf16x4*)((bf16_t*)out + (size_t)place * (N >> 1) + (f >> 1)) = o;
        }
    }
}

// Prompts.  A block takes 256 features of one tile (TT * 32 rows): operand tiles of both matrices go from memory straight
// into LDS (global_load_lds_dwordx4), through a ring of NS stages of 32 k with one barrier each, as in the tiled
// product; the rows are gathered by the lanes' own addresses.  Four waves, two along the features and two along the rows,
// 8 x TT accumulator tiles each.  Blocks are dealt to the eight dies in runs of equal length over the tiles that are in
// use; neighbours in a run are tiles of the same features, up to four of them, which mostly belong to one expert and
// read the same weights.
#define MP_FEATURES 256
#define MP_GROUP 4
template <int TT, int NS, int GATE>
__global__ __launch_bounds__(256, 2) void moe_packed_kernel(const bf16_t* __restrict__ x, const int* __restrict__ src_row,
                                                            const float* __restrict__ src_scale, const bf16_t* __restrict__ wp,
                                                            void* __restrict__ out, const int* __restrict__ tiles, int max_tiles,
                                                            int N, int K, MoeGate mg) {
    constexpr int FT = 8, NTF = 16, NTT = 2 * TT, TILES = NTF + NTT, LW = NTF / 4, LX = (NTT + 3) / 4, LPS = LW + LX;
    static_assert(NTT % 4 == 0, "the row tiles divide among the waves");
    extern __shared__ __attribute__((aligned(16))) bf16_t ring[];          // [NS][TILES][512]
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int wf = wave & 1, wt = wave >> 1;
    int used = 0;                                                         // tiles with rows come first
    for (int t = 0; t < max_tiles; t += 256) used += __syncthreads_count(t + tid < max_tiles && tiles[4 * (t + tid) + 2] > 0);
    const int n_ft = (N + MP_FEATURES - 1) / MP_FEATURES;
    const int total = n_ft * used, per_die = (total + 7) >> 3;
    const int lin = (blockIdx.x & 7) * per_die + (blockIdx.x >> 3);
    if ((int)(blockIdx.x >> 3) >= per_die || lin >= total) return;
    const int grp = lin / (MP_GROUP * n_ft), within = lin - grp * (MP_GROUP * n_ft);
    const int gt = min(MP_GROUP, used - grp * MP_GROUP);
    const int tile = grp * MP_GROUP + within % gt, n0 = (within / gt) * MP_FEATURES;
    const int e = tiles[4 * tile], p0 = tiles[4 * tile + 1], M = tiles[4 * tile + 2];
    if (e < 0) return;                                                    // (an identity expert's)
    const int n_steps = K >> 5, n_groups = N >> 4;
    f32x4 acc[FT][TT];
#pragma unroll
    for (int a = 0; a < FT; ++a)
#pragma unroll
        for (int b = 0; b < TT; ++b) acc[a][b] = (f32x4){0.f, 0.f, 0.f, 0.f};
    const bf16_t* we = wp + (size_t)e * N * K;
    const bf16_t *wsrc[LW], *xsrc[LX];
#pragma unroll
    for (int u = 0; u < LW; ++u) wsrc[u] = we + ((size_t)min((n0 >> 4) + wave * LW + u, n_groups - 1) * n_steps * 64 + lane) * 8;
    // four lanes per row of 64 bytes, its pieces exchanged by (row / 2) % 4 so that the operand reads meet no bank twice
    const int x_piece = 8 * ((lane & 3) ^ ((lane >> 3) & 3));
#pragma unroll
    for (int u = 0; u < LX; ++u) {
        const int p = p0 + min((wave * LX + u) * 16 + (lane >> 2), M - 1);
        xsrc[u] = x + (size_t)(src_row ? src_row[p] : p) * K + x_piece;
    }
    const int x_read = 32 * (lane & 15) + 8 * ((lane >> 4) ^ (((lane & 15) >> 1) & 3));
    auto issue = [&](int i) {
        bf16_t* slot = ring + (size_t)(i % NS) * TILES * 512;
#pragma unroll
        for (int u = 0; u < LW; ++u) {
            __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)wsrc[u],
                                             (__attribute__((address_space(3))) void*)(slot + (wave * LW + u) * 512), 16, 0, 0);
            wsrc[u] += 512;
        }
#pragma unroll
        for (int u = 0; u < LX; ++u) {
            __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)xsrc[u],
                                             (__attribute__((address_space(3))) void*)(slot + (NTF + wave * LX + u) * 512), 16, 0, 0);
            xsrc[u] += 32;
        }
    };
#pragma unroll
    for (int i = 0; i < NS - 1; ++i)
        if (i < n_steps) issue(i);
    for (int i = 0; i < n_steps; ++i) {
        // my loads of this stage have landed when at most the later stages' are in flight
        constexpr int LATER = LPS * (NS - 2);
        if (i + NS - 2 < n_steps) __builtin_amdgcn_s_waitcnt(0xF70 | (LATER & 0xF) | (((LATER >> 4) & 3) << 14));
        else __builtin_amdgcn_s_waitcnt(0xF70);
        asm volatile("s_barrier" ::: "memory");                           // (a bare one: __syncthreads would wait for all loads)
        const bf16_t* slot = ring + (size_t)(i % NS) * TILES * 512;
        bf16x8 a[FT], b[TT];
#pragma unroll
        for (int t = 0; t < TT; ++t) b[t] = *(const bf16x8*)(slot + (NTF + wt * TT + t) * 512 + x_read);
#pragma unroll
        for (int t = 0; t < FT; ++t) a[t] = *(const bf16x8*)(slot + (wf * FT + t) * 512 + lane * 8);
        __builtin_amdgcn_sched_barrier(0);
        if (i + NS - 1 < n_steps) issue(i + NS - 1);
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int ta = 0; ta < FT; ++ta)
#pragma unroll
            for (int tb = 0; tb < TT; ++tb) acc[ta][tb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[ta], b[tb], acc[ta][tb], 0, 0, 0);
    }
    const int j = lane & 15, g = lane >> 4;
#pragma unroll
    for (int tb = 0; tb < TT; ++tb) {
        const int r = (wt * TT + tb) * 16 + j;
        if (r >= M) continue;                                             // (the same for the four lanes of a row)
        const float scale = src_scale ? src_scale[p0 + r] : 1.0f;
#pragma unroll
        for (int ta = 0; ta < FT; ++ta) moe_store<GATE>(mg, out, p0 + r, n0 + (wf * FT + ta) * 16 + 4 * g, g, acc[ta][tb] * scale, N);
    }
}

#define MS_FEATURES 32        // features per block of the streaming form
#define MS_ROWS 64
// Steps of few rows (decoding), where nearly every tile holds a row or two and all a block does is stream its expert's
// weights: a block takes 32 features and its four waves deal the steps of K out among them (wave w: steps w, w + 4, ...),
// so that even a step that touches four experts has some hundred blocks; their sums are added through LDS in a fixed
// order.  No barrier inside the loop.
template <int GATE>
__global__ __launch_bounds__(256) void moe_packed_stream_kernel(const bf16_t* __restrict__ x, const int* __restrict__ src_row,
                                                                const float* __restrict__ src_scale, const bf16_t* __restrict__ wp,
                                                                void* __restrict__ out, const int* __restrict__ tiles, int N, int K,
                                                                MoeGate mg) {
    __shared__ f32x4 part[4][2][4][64];
    const int e = tiles[4 * blockIdx.y + 0];
    if (e < 0) return;
    const int p0 = tiles[4 * blockIdx.y + 1], M = tiles[4 * blockIdx.y + 2];
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int col = lane & 15, g = lane >> 4;
    const int f0 = blockIdx.x * MS_FEATURES;
    const int n_steps = K >> 5, n_groups = N >> 4;
    const bf16_t* wrow[2];
#pragma unroll
    for (int a = 0; a < 2; ++a)
        wrow[a] = wp + (size_t)e * N * K + ((size_t)min((f0 >> 4) + a, n_groups - 1) * n_steps * 64 + lane) * 8;
    const int groups = (M + 15) >> 4;
    const bf16_t* xrow[4];
#pragma unroll
    for (int t = 0; t < 4; ++t) {
        const int p = p0 + min(16 * t + col, M - 1);                      // (rows beyond the tile: any row, nobody reads their sums)
        xrow[t] = x + (size_t)(src_row ? src_row[p] : p) * K + 8 * g;
    }
    f32x4 acc[2][4];
#pragma unroll
    for (int a = 0; a < 2; ++a)
#pragma unroll
        for (int t = 0; t < 4; ++t) acc[a][t] = (f32x4){0.f, 0.f, 0.f, 0.f};
    auto walk = [&](auto n) {                                             // (the number of row groups is chosen once, outside the loop)
        constexpr int G = decltype(n)::value;
#pragma unroll 8
        for (int s = wave; s < n_steps; s += 4) {
            bf16x8 av[2], bv[G];
#pragma unroll
            for (int a = 0; a < 2; ++a) av[a] = *(const bf16x8*)(wrow[a] + (size_t)s * 512);
#pragma unroll
            for (int t = 0; t < G; ++t) bv[t] = *(const bf16x8*)(xrow[t] + 32 * s);
#pragma unroll
            for (int t = 0; t < G; ++t)
#pragma unroll
                for (int a = 0; a < 2; ++a) acc[a][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(av[a], bv[t], acc[a][t], 0, 0, 0);
        }
    };
    if (groups <= 1) walk(std::integral_constant<int, 1>{});
    else walk(std::integral_constant<int, 4>{});
#pragma unroll
    for (int a = 0; a < 2; ++a)
#pragma unroll
        for (int t = 0; t < 4; ++t)
            if (t < groups) part[wave][a][t][lane] = acc[a][t];
    __syncthreads();
    if (wave != 0) return;
#pragma unroll
    for (int t = 0; t < 4; ++t) {
        const int r = 16 * t + col;
        if (r >= M) continue;
        const float scale = src_scale ? src_scale[p0 + r] : 1.0f;
#pragma unroll
        for (int a = 0; a < 2; ++a) {
            const f32x4 sum = (part[0][a][t][lane] + part[1][a][t][lane]) + (part[2][a][t][lane] + part[3][a][t][lane]);
            moe_store<GATE>(mg, out, p0 + r, f0 + 16 * a + 4 * g, g, sum * scale, N);
        }
    }
}

extern "C" int fl_moe_packed_takes(int N, int K) { return N > 0 && N % 16 == 0 && K > 0 && K % 32 == 0; }

template <int TT, int GATE>
static int launch_moe_packed(const void* x, const int* src_row, const float* src_scale, const void* w, void* out, const int* tiles,
                             int max_tiles, int N, int K, MoeGate mg, hipStream_t stream) {
    constexpr int NS = 3, LDS = NS * (16 + 2 * TT) * 1024;
    static bool sized = false;
    if (!sized) {
        hipError_t e_ = hipFuncSetAttribute((const void*)moe_packed_kernel<TT, NS, GATE>, hipFuncAttributeMaxDynamicSharedMemorySize, LDS);
        FL_CHECK(e_ == hipSuccess, "moe_packed: %s", hipGetErrorString(e_));
        sized = true;
    }
    const long blocks = (long)ceil_div(N, MP_FEATURES) * max_tiles;
    FL_CHECK(blocks < (1L << 30), "moe_packed: too many row tiles");
    moe_packed_kernel<TT, NS, GATE><<<(unsigned)((blocks + 7) / 8 * 8), 256, LDS, stream>>>((const bf16_t*)x, src_row, src_scale, (const bf16_t*)w, out, tiles, max_tiles, N, K, mg);
    return 0;
}

extern "C" int fl_moe_packed(const void* x, const int* src_row, const float* src_scale, const void* w, void* out, const int* tiles,
                             int max_tiles, int tile_rows, int n_rows, int N, int K, int gate, float alpha, float limit,
                             float shift, hipStream_t stream) {
    FL_CHECK(max_tiles >= 0 && n_rows >= 0 && fl_moe_packed_takes(N, K), "moe_packed: %d features over %d values are not taken", N, K);
    FL_CHECK((uintptr_t)x % 16 == 0 && (uintptr_t)w % 16 == 0 && (uintptr_t)out % 16 == 0, "moe_packed: operands must be 16-byte aligned");
    FL_CHECK(tile_rows == 64 || tile_rows == 128, "moe_packed: tiles of %d rows (64 or 128)", tile_rows);
    FL_CHECK(gate >= MG_NONE && gate <= MG_CLAMPED, "moe_packed: unknown gate %d", gate);
    if (max_tiles == 0) return 0;
    const MoeGate mg = {alpha, limit, shift};
    if (n_rows <= 2 * MS_ROWS && tile_rows == MS_ROWS) {
        FL_CHECK(max_tiles <= 65535, "moe_packed: %d row tiles are more than one grid takes", max_tiles);
        dim3 grid(ceil_div(N, MS_FEATURES), max_tiles);
#define FL_MS(G) moe_packed_stream_kernel<G><<<grid, 256, 0, stream>>>((const bf16_t*)x, src_row, src_scale, (const bf16_t*)w, out, tiles, N, K, mg)
        if (gate == MG_NONE) FL_MS(MG_NONE);
        else if (gate == MG_SILU) FL_MS(MG_SILU);
        else FL_MS(MG_CLAMPED);
#undef FL_MS
    } else {
#define FL_MP(TT, G) launch_moe_packed<TT, G>(x, src_row, src_scale, w, out, tiles, max_tiles, N, K, mg, stream)
        int rc;
        if (tile_rows == 128) rc = gate == MG_NONE ? FL_MP(4, MG_NONE) : gate == MG_SILU ? FL_MP(4, MG_SILU) : FL_MP(4, MG_CLAMPED);
        else rc = gate == MG_NONE ? FL_MP(2, MG_NONE) : gate == MG_SILU ? FL_MP(2, MG_SILU) : FL_MP(2, MG_CLAMPED);
#undef FL_MP
        if (rc != 0) return rc;
    }
    FL_LAUNCH_CHECK();
    return 0;
}
FL_RECORDABLE(fl_moe_packed)

// ------------------------------------------------------------------ a product with few output features
// out[m][f] = sum_k x[m][k] w[f][k] for a handful of features (a router's scores, a gate's logit): one
// wave per row and FF neighbouring features (many rows: four, so that a row is read less often; few: one), the lanes
// stride over k and add their parts in a fixed tree, so an element does not depend on how many rows the call
// has.  Products of stored values are exact in float; the sums are float.
template <typename T, int FF>
__global__ __launch_bounds__(256) void gemm_few_kernel(const T* __restrict__ x, const T* __restrict__ w, float* __restrict__ out,
                                                       long total, int N, int K) {
    const long unit = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (unit >= total) return;
    const int lane = threadIdx.x & 63;
    const int per_row = (N + FF - 1) / FF;
    const long m = unit / per_row;
    const int f = (int)(unit - m * per_row) * FF;
    const T* xr = x + (size_t)m * K;
    const T* wr[FF];
#pragma unroll
    for (int q = 0; q < FF; ++q) wr[q] = w + (size_t)min(f + q, N - 1) * K;
    float a[FF][4];
#pragma unroll
    for (int q = 0; q < FF; ++q)
#pragma unroll
        for (int r = 0; r < 4; ++r) a[q][r] = 0.f;
    int k = 4 * lane;
    if (K % 4 == 0) {
        for (; k + 3 < K; k += 256) {
            float xv[4];
#pragma unroll
            for (int r = 0; r < 4; ++r) xv[r] = to_f32(xr[k + r]);
#pragma unroll
            for (int q = 0; q < FF; ++q)
#pragma unroll
                for (int r = 0; r < 4; ++r) a[q][r] = fmaf(xv[r], to_f32(wr[q][k + r]), a[q][r]);
        }
    } else {
        for (k = lane; k < K; k += 64)
#pragma unroll
            for (int q = 0; q < FF; ++q) a[q][0] = fmaf(to_f32(xr[k]), to_f32(wr[q][k]), a[q][0]);
    }
#pragma unroll
    for (int q = 0; q < FF; ++q) {
        const float s = wave_sum((a[q][0] + a[q][1]) + (a[q][2] + a[q][3]));
        if (lane == 0 && f + q < N) out[m * N + f + q] = s;
    }
}

extern "C" int fl_gemm_few(const void* x, const void* w, float* out, int dtype, int M, int N, int K, hipStream_t stream) {
    FL_CHECK(M >= 0 && N > 0 && K > 0, "gemm_few: bad sizes M=%d N=%d K=%d", M, N, K);
    if (M == 0) return 0;
    const bool many = M >= 64;
    const long total = (long)M * (many ? ceil_div(N, 4) : N);
    const long blocks = (total + 3) / 4;
    FL_CHECK(blocks < (1L << 31), "gemm_few: too many outputs");
#define FL_GF(T, FF) gemm_few_kernel<T, FF><<<(unsigned)blocks, 256, 0, stream>>>((const T*)x, (const T*)w, out, total, N, K)
    if (dtype == FL_F32) { if (many) FL_GF(float, 4); else FL_GF(float, 1); }
    else if (dtype == FL_BF16) { if (many) FL_GF(bf16_t, 4); else FL_GF(bf16_t, 1); }
#undef FL_GF
    else FL_CHECK(false, "gemm_few: unknown dtype %d", dtype);
    FL_LAUNCH_CHECK();
    return 0;
}
FL_RECORDABLE(fl_gemm_few)
