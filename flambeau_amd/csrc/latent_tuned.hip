// Attention over cached latent rows on the matrix cores (bfloat16 pools), and the small products per
// head around it.
//
// A wave takes one token and up to 16 of its heads; every head of a token sees the same rows, so a
// loaded row serves all 16.  Everything is computed transposed, as in the other attention kernels of
// this library: S^T[key][head] = C[key][:] . Qa[head][:] (A = rows of the page, B = the folded queries,
// held in registers for the whole walk) and Z^T[dim][head] += C^T[dim][key] P^T[key][head] (A = the
// page's transposed copy, B = the weights, which are the lanes' own score accumulators: the rows of
// the score tiles are dealt out so that a lane's eight values of two tiles are eight keys in a row).
// A head is a lane column, so maxima, sums and rescaling need no broadcast.  Waves share nothing:
// rows of different requests may lie in one block.  Keys beyond the query's position are given weight
// zero and their values are set to zero before they are multiplied, so what an unused or reused page
// holds (a NaN too) never reaches a sum.
//
// A row is K values wide as a key and R as a value (its first R values; K > R where a rotated key part stands behind
// the latent); folded queries are K wide, the weighted sums R.
// sink (float [H], or null): a score per head that joins the denominator once, not scaled, with no key and no value.
//
// A kernel is compiled for the most steps of 32 values it takes and runs that many whatever K and R are: a step beyond
// K multiplies zeros of the query with the row's first values, one beyond R fills sums that nobody reads.  A branch
// around a load would make the compiler wait for every load before it issues the next.
#include "common.h"
#include "api.h"
#include "recordable.h"
#include "query_tail.h"

#define LT_WAVES 4
#define LT_CHUNK 64

// v with the values of the keys outside first_visible .. last_visible set to zero (v holds eight keys from first_key on)
__device__ __forceinline__ bf16x8 keep_keys(bf16x8 v, int first_key, int first_visible, int last_visible) {
#pragma unroll
    for (int e = 0; e < 8; ++e)
        v[e] = first_key + e > last_visible || first_key + e < first_visible ? (bf16_t)0.f : v[e];
    return v;
}

// qa: bfloat16 [n][H][K]; z: float [n][H][R]; pool: [n_pages][page_size * (K + R)]; K = 32 * nk, nk <= NK, R = 32 * ns, ns <= NS.
// n_split > 1: the keys of every token are dealt out to that many waves, which leave their sums in
// part_o [n * groups * n_split * 16][R] and (maximum, sum of weights) in part_ml [...][2]; a second kernel adds them.
template <int NK, int NS>
__global__ __launch_bounds__(64 * LT_WAVES) void latent_attention_mfma_kernel(
    const bf16_t* __restrict__ qa, float* __restrict__ z, const bf16_t* __restrict__ pool,
    const int* __restrict__ positions, const int* __restrict__ tok_seq, const int* __restrict__ block_table,
    int max_blocks, int n, int H, int K, int R, int page_size, int n_pages, float scale, int window, int groups_per_token,
    int n_split, float* __restrict__ part_o, float* __restrict__ part_ml, const float* __restrict__ sink) {
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int unit = blockIdx.x * LT_WAVES + wave;                 // (token, group of 16 heads, part of the keys)
    if (unit >= n * groups_per_token * n_split) return;
    const int split = unit % n_split, tg = unit / n_split;
    const int token = tg / groups_per_token, h0 = (tg - token * groups_per_token) * 16;
    const int col = lane & 15, g = lane >> 4;                      // col: head (B columns) or row of an A tile
    const int nk = K >> 5, ns = R >> 5;
    const int p = positions[token];
    const int* table = block_table + (size_t)tok_seq[token] * max_blocks;
    const int lo = window > 0 ? max(0, p - window + 1) : 0;
    const size_t page_stride = (size_t)page_size * (K + R);
    const bool head_live = h0 + col < H;

    // the folded queries of this lane's head: B operand of every score product
    bf16x8 qreg[NK];
    {
        const bf16_t* qr = qa + ((size_t)token * H + h0 + (head_live ? col : 0)) * K;
#pragma unroll
        for (int s = 0; s < NK; ++s) {
            if (s < nk && head_live) {
                qreg[s] = *(const bf16x8*)(qr + 32 * s + 8 * g);
            } else {
#pragma unroll
                for (int e = 0; e < 8; ++e) qreg[s][e] = (bf16_t)0.f;
            }
        }
    }
    f32x4 o[2 * NS];                                               // Z^T tiles: dims 16 t + 4 g + r of head `col`
#pragma unroll
    for (int t = 0; t < 2 * NS; ++t) o[t] = (f32x4){0.f, 0.f, 0.f, 0.f};
    float m = -INFINITY, l = 0.f;

    int first = lo & ~(LT_CHUNK - 1);                              // chunks are aligned, so a tile of 16 keys lies in one page
    int last = p;
    if (n_split > 1) {
        // this part's chunks: the token's chunks dealt out in equal runs (a short context leaves late parts empty)
        const int chunks = (p - first) / LT_CHUNK + 1, per = (chunks + n_split - 1) / n_split;
        last = min(p, first + (split + 1) * per * LT_CHUNK - 1);
        first += split * per * LT_CHUNK;
    }
    for (int t0 = first; t0 <= last; t0 += LT_CHUNK) {
        // ---- scores of 64 keys: four tiles of 16; tile 2 q + b, row i <-> key t0 + 32 q + 8 (i / 4) + 4 b + i % 4
        f32x4 sacc[4];
#pragma unroll
        for (int a = 0; a < 4; ++a) {
            sacc[a] = (f32x4){0.f, 0.f, 0.f, 0.f};
            const int key = t0 + 32 * (a >> 1) + 8 * (col >> 2) + 4 * (a & 1) + (col & 3);
            const int kc = min(key, p);                            // a key beyond p: any loadable row, masked below
            int page = table[kc / page_size];
            page = min(max(page, 0), n_pages - 1);
            const bf16_t* row = pool + (size_t)page * page_stride + (size_t)(kc % page_size) * K + 8 * g;
#pragma unroll
            for (int s = 0; s < NK; ++s)
                sacc[a] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*(const bf16x8*)(row + (s < nk ? 32 * s : 0)), qreg[s], sacc[a], 0, 0, 0);
        }
        // lane (head col, g): sacc[2 q + b][e] is key t0 + 32 q + 8 g + 4 b + e
        float cmax = -INFINITY;
#pragma unroll
        for (int a = 0; a < 4; ++a)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int key = t0 + 32 * (a >> 1) + 8 * g + 4 * (a & 1) + e;
                sacc[a][e] = key > p || key < lo ? -INFINITY : sacc[a][e] * scale;
                cmax = fmaxf(cmax, sacc[a][e]);
            }
        cmax = fmaxf(cmax, __shfl_xor(cmax, 16, FL_WAVE));
        cmax = fmaxf(cmax, __shfl_xor(cmax, 32, FL_WAVE));
        const float m_new = fmaxf(m, cmax);                        // finite: every chunk holds a visible key
        const float corr = expf(m - m_new);
        m = m_new;
        bf16x8 pb[2];
        float lsum = 0.f;
#pragma unroll
        for (int a = 0; a < 4; ++a)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const bf16_t w = (bf16_t)expf(sacc[a][e] - m_new);
                pb[a >> 1][4 * (a & 1) + e] = w;
                lsum += (float)w;                                  // the sum of the weights as they are multiplied
            }
        lsum += __shfl_xor(lsum, 16, FL_WAVE);
        lsum += __shfl_xor(lsum, 32, FL_WAVE);
        l = l * corr + lsum;
        // ---- weighted sum: Z^T[dim][head] += C^T[dim][keys] P^T[keys][head], 32 keys a step
        const bool edge = t0 + LT_CHUNK - 1 > p || t0 < lo;
        const bf16_t* cols[2];
        int key0[2];
#pragma unroll
        for (int q = 0; q < 2; ++q) {
            key0[q] = t0 + 32 * q + 8 * g;
            const int kc = min(key0[q], p);
            int page = table[kc / page_size];
            page = min(max(page, 0), n_pages - 1);
            cols[q] = pool + (size_t)page * page_stride + (size_t)page_size * K + (key0[q] % page_size);
        }
#pragma unroll
        for (int t = 0; t < 2 * NS; ++t) {
            o[t] *= corr;
#pragma unroll
            for (int q = 0; q < 2; ++q) {
                bf16x8 v = *(const bf16x8*)(cols[q] + (size_t)((t < 2 * ns ? 16 * t : 0) + col) * page_size);
                if (edge) v = keep_keys(v, key0[q], lo, p);
                o[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, pb[q], o[t], 0, 0, 0);
            }
        }
    }
    if (n_split > 1) {
        // unnormalised sums relative to this part's own maximum; fl_latent_attention_mfma's second kernel adds the parts
        float* po = part_o + ((size_t)unit * 16 + col) * R;
#pragma unroll
        for (int t = 0; t < 2 * NS; ++t)
            if (t < 2 * ns) *(f32x4*)(po + 16 * t + 4 * g) = o[t];
        if (g == 0) {
            part_ml[((size_t)unit * 16 + col) * 2] = m;
            part_ml[((size_t)unit * 16 + col) * 2 + 1] = l;
        }
        return;
    }
    if (!head_live) return;
    const float inv = sink ? softmax_factor_with_sink(m, l, sink[h0 + col]) : l > 0.f ? 1.0f / l : 0.f;
    float* zr = z + ((size_t)token * H + h0 + col) * R;
#pragma unroll
    for (int t = 0; t < 2 * NS; ++t)
        if (t < 2 * ns) *(f32x4*)(zr + 16 * t + 4 * g) = o[t] * inv;
}

// z[token][head][:] = sum_s o_s exp(m_s - M) / sum_s l_s exp(m_s - M), M = max_s m_s, over the parts of the keys
// (rising s; an empty part left zeros and has weight 0).  A block takes 256 dims of one (token, head): its
// first wave makes the parts' weights, then every thread adds its dim's parts, all loads independent.
__global__ __launch_bounds__(256) void latent_merge_kernel(const float* __restrict__ part_o, const float* __restrict__ part_ml,
                                                           float* __restrict__ z, int H, int R, int groups, int n_split,
                                                           const float* __restrict__ sink) {
    __shared__ float ws[64];
    __shared__ float inv_l;
    const int unit = blockIdx.x, d = blockIdx.y * 256 + threadIdx.x;
    const int token = unit / H, h = unit - token * H;
    const size_t base = ((size_t)(token * groups + (h >> 4)) * n_split) * 16 + (h & 15);        // part 0; parts are 16 rows apart
    if (threadIdx.x < 64) {
        const int lane = threadIdx.x;
        const float ms = lane < n_split ? part_ml[(base + (size_t)lane * 16) * 2] : -INFINITY;
        const float ls = lane < n_split ? part_ml[(base + (size_t)lane * 16) * 2 + 1] : 0.f;
        const float M = wave_max(ms);
        const float w = ms > -INFINITY ? expf(ms - M) : 0.f;
        const float L = wave_sum(ls * w);
        ws[lane] = w;
        if (lane == 0) inv_l = sink ? softmax_factor_with_sink(M, L, sink[h]) : L > 0.f ? 1.0f / L : 0.f;
    }
    __syncthreads();
    if (d >= R) return;
    float acc = 0.f;
#pragma unroll 8
    for (int s = 0; s < n_split; ++s) acc = fmaf(part_o[(base + (size_t)s * 16) * R + d], ws[s], acc);
    z[(size_t)unit * R + d] = acc * inv_l;
}

// Whether the kernels take a pool's shape: values of a multiple of 32 up to 512, keys as wide or one or two steps of
// 32 wider, pages of a multiple of 16 rows.
extern "C" int fl_latent_attention_mfma_takes(int K, int R, int page_size) {
    return R > 0 && R % 32 == 0 && R <= 512 && K % 32 == 0 && K >= R && K <= R + 64 && page_size > 0 && page_size % 16 == 0;
}

extern "C" int fl_latent_attention_mfma(const void* qa, float* z, const void* pool, const int* positions,
                                        const int* tok_seq, const int* block_table, int max_blocks, int n, int H, int K, int R,
                                        int page_size, int n_pages, float scale, int window, int n_split, float* part_o,
                                        float* part_ml, const float* sink, hipStream_t stream) {
    FL_CHECK(n >= 0 && H > 0 && n_pages > 0 && max_blocks > 0, "latent_attention_mfma: bad sizes");
    FL_CHECK(n_split >= 1 && n_split <= 64 && (n_split == 1 || (part_o && part_ml)), "latent_attention_mfma: %d parts of the keys (at most 64) need a workspace", n_split);
    FL_CHECK(fl_latent_attention_mfma_takes(K, R, page_size), "latent_attention_mfma: rows of %d and %d values in pages of %d are not taken", K, R, page_size);
    FL_CHECK((uintptr_t)qa % 16 == 0 && (uintptr_t)pool % 16 == 0 && (uintptr_t)z % 16 == 0, "latent_attention_mfma: operands must be 16-byte aligned");
    FL_CHECK(window >= 0, "latent_attention_mfma: negative window");
    if (n == 0) return 0;
    const int groups = ceil_div(H, 16);
    const long units = (long)n * groups * n_split;
    FL_CHECK(units < (1L << 30), "latent_attention_mfma: too many rows");
    const int blocks = (int)((units + LT_WAVES - 1) / LT_WAVES);
    const int ns = R / 32;
#define FL_LT(NK, NS)                                                                                                       \
    latent_attention_mfma_kernel<NK, NS><<<blocks, 64 * LT_WAVES, 0, stream>>>((const bf16_t*)qa, z, (const bf16_t*)pool,  \
                                                                           positions, tok_seq, block_table, max_blocks, \
                                                                           n, H, K, R, page_size, n_pages, scale, window, groups, \
                                                                           n_split, part_o, part_ml, sink)
    if (K == R) {
        if (ns <= 2) FL_LT(2, 2);
        else if (ns <= 4) FL_LT(4, 4);
        else if (ns <= 8) FL_LT(8, 8);
        else FL_LT(16, 16);
    } else {
        if (ns <= 2) FL_LT(4, 2);
        else if (ns <= 4) FL_LT(6, 4);
        else if (ns <= 8) FL_LT(10, 8);
        else FL_LT(18, 16);
    }
#undef FL_LT
    FL_LAUNCH_CHECK();
    if (n_split > 1) {
        dim3 mgrid(n * H, ceil_div(R, 256));
        latent_merge_kernel<<<mgrid, 256, 0, stream>>>(part_o, part_ml, z, H, R, groups, n_split, sink);
        FL_LAUNCH_CHECK();
    }
    return 0;
}
FL_RECORDABLE(fl_latent_attention_mfma)


// The same walk for prompt portions, four waves to a block that share their keys: a tile (from the host:
// first token, tokens, first group of 16 heads, groups; tokens x groups <= 4, all of one request) loads
// every chunk of 64 rows once into LDS, as it is and transposed, and its waves read their operands from
// there.  Without this every wave fetches every row itself and the kernel runs at the rate of the
// caches, 16 flops a byte.  Rows are padded by 16 bytes so that the 16 rows (or dims) of an operand
// start in different banks.  A wave whose token lies before a chunk sits the chunk out.
template <int NK, int NS>
__global__ __launch_bounds__(64 * LT_WAVES) void latent_attention_shared_kernel(
    const bf16_t* __restrict__ qa, float* __restrict__ z, const bf16_t* __restrict__ pool,
    const int* __restrict__ positions, const int* __restrict__ tok_seq, const int* __restrict__ block_table,
    int max_blocks, int H, int K, int R, int page_size, int n_pages, float scale, int window, const int* __restrict__ tiles,
    const float* __restrict__ sink) {
    extern __shared__ __attribute__((aligned(16))) unsigned char lt_smem[];
    const int stride_r = K + 8, stride_c = LT_CHUNK + 8;
    bf16_t* ks = (bf16_t*)lt_smem;                                  // [64 keys][K + 8]
    bf16_t* vs = ks + (size_t)LT_CHUNK * stride_r;                  // [R dims][64 + 8]
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int t_first = tiles[4 * blockIdx.x], n_tok = tiles[4 * blockIdx.x + 1];
    const int g_first = tiles[4 * blockIdx.x + 2], n_grp = tiles[4 * blockIdx.x + 3];
    const int tw = wave / n_grp, gw = wave - tw * n_grp;
    const bool active = tw < n_tok;
    const int token = t_first + (active ? tw : 0), h0 = (g_first + gw) * 16;
    const int col = lane & 15, g = lane >> 4;
    const int nk = K >> 5, ns = R >> 5;
    const int p = active ? positions[token] : -1;
    const int p_max = positions[t_first + n_tok - 1];              // a request's tokens of a step stand in rising order
    const int* table = block_table + (size_t)tok_seq[t_first] * max_blocks;
    const int lo = window > 0 ? max(0, p - window + 1) : 0;
    const int lo_min = window > 0 ? max(0, positions[t_first] - window + 1) : 0;
    const size_t page_stride = (size_t)page_size * (K + R);
    const bool head_live = active && h0 + col < H;
    bf16x8 qreg[NK];
    {
        const bf16_t* qr = qa + ((size_t)token * H + (head_live ? h0 + col : 0)) * K;
#pragma unroll
        for (int s = 0; s < NK; ++s) {
            if (s < nk && head_live) {
                qreg[s] = *(const bf16x8*)(qr + 32 * s + 8 * g);
            } else {
#pragma unroll
                for (int e = 0; e < 8; ++e) qreg[s][e] = (bf16_t)0.f;
            }
        }
    }
    f32x4 o[2 * NS];
#pragma unroll
    for (int t = 0; t < 2 * NS; ++t) o[t] = (f32x4){0.f, 0.f, 0.f, 0.f};
    float m = -INFINITY, l = 0.f;
    const int pieces_r = K >> 3;                                    // 16-byte pieces of a row
    for (int t0 = lo_min & ~(LT_CHUNK - 1); t0 <= p_max; t0 += LT_CHUNK) {
        // ---- the chunk into LDS: rows as they are, and the pages' transposed copies dim by dim.  The pages of the
        // chunk's four runs of 16 keys are looked up first (pages hold a multiple of 16 rows), so that all copies
        // of a thread are in flight at once; a run beyond the newest token takes that token's page and is masked.
        const bf16_t* run_rows[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int kc = min(t0 + 16 * j, p_max & ~15);
            int page = table[kc / page_size];
            page = min(max(page, 0), n_pages - 1);
            run_rows[j] = pool + (size_t)page * page_stride + (size_t)(kc % page_size) * K;       // row kc of the page; the transposed values begin behind the page's page_size rows
        }
#pragma unroll
        for (int i = 0; i < 16; ++i) {                             // wave w copies rows w, w + 4, ...: row 4 i + w lies in run i / 4
            const int row = 4 * i + wave;
            const bf16_t* src = run_rows[i >> 2] + (size_t)(row & 15) * K;
            for (int c = lane; c < pieces_r; c += 64) *(bf16x8*)(ks + (size_t)row * stride_r + 8 * c) = *(const bf16x8*)(src + 8 * c);
        }
        {
            const int k8 = threadIdx.x & 7;                        // this thread's 8 keys of every dim: run k8 / 2, its first or second half
            const int kc = min(t0 + 16 * (k8 >> 1), p_max & ~15);
            const bf16_t* src = run_rows[0];
#pragma unroll
            for (int j = 1; j < 4; ++j) src = (k8 >> 1) == j ? run_rows[j] : src;
            src += (size_t)(page_size - (kc % page_size)) * K + (kc % page_size) + 8 * (k8 & 1);    // from row kc of the page to column kc (+ 8) of its transposed copy
            for (int dim = threadIdx.x >> 3; dim < R; dim += 32)
                *(bf16x8*)(vs + (size_t)dim * stride_c + 8 * k8) = *(const bf16x8*)(src + (size_t)dim * page_size);
        }
        __syncthreads();
        if (active && t0 <= p && t0 + LT_CHUNK - 1 >= lo) {
            f32x4 sacc[4];
#pragma unroll
            for (int a = 0; a < 4; ++a) {
                sacc[a] = (f32x4){0.f, 0.f, 0.f, 0.f};
                const bf16_t* row = ks + (size_t)(32 * (a >> 1) + 8 * (col >> 2) + 4 * (a & 1) + (col & 3)) * stride_r + 8 * g;
#pragma unroll
                for (int s = 0; s < NK; ++s)
                    sacc[a] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*(const bf16x8*)(row + (s < nk ? 32 * s : 0)), qreg[s], sacc[a], 0, 0, 0);
            }
            float cmax = -INFINITY;
#pragma unroll
            for (int a = 0; a < 4; ++a)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const int key = t0 + 32 * (a >> 1) + 8 * g + 4 * (a & 1) + e;
                    sacc[a][e] = key > p || key < lo ? -INFINITY : sacc[a][e] * scale;
                    cmax = fmaxf(cmax, sacc[a][e]);
                }
            cmax = fmaxf(cmax, __shfl_xor(cmax, 16, FL_WAVE));
            cmax = fmaxf(cmax, __shfl_xor(cmax, 32, FL_WAVE));
            // The base of the exponents follows the maximum lazily: it moves only when a score exceeds it by more
            // than 8 (weights stay below e^8, exact enough in bfloat16 and float), so that in most chunks nothing
            // is rescaled and the sums can stay where the matrix cores accumulate them.
            const float m_new = (cmax > m + 8.0f) ? cmax : m;      // finite after the first chunk: it holds a key this wave sees
            const bool moved = __any(m_new != m);
            const float corr = expf(m - m_new);
            m = m_new;
            bf16x8 pb[2];
            float lsum = 0.f;
#pragma unroll
            for (int a = 0; a < 4; ++a)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const bf16_t w = (bf16_t)expf(sacc[a][e] - m_new);
                    pb[a >> 1][4 * (a & 1) + e] = w;
                    lsum += (float)w;
                }
            lsum += __shfl_xor(lsum, 16, FL_WAVE);
            lsum += __shfl_xor(lsum, 32, FL_WAVE);
            l = l * corr + lsum;
            if (moved) {
#pragma unroll
                for (int t = 0; t < 2 * NS; ++t) o[t] *= corr;
            }
            const bool edge = t0 + LT_CHUNK - 1 > p || t0 < lo;
#pragma unroll
            for (int t = 0; t < 2 * NS; ++t) {
#pragma unroll
                for (int q = 0; q < 2; ++q) {
                    bf16x8 v = *(const bf16x8*)(vs + (size_t)((t < 2 * ns ? 16 * t : 0) + col) * stride_c + 32 * q + 8 * g);
                    if (edge) v = keep_keys(v, t0 + 32 * q + 8 * g, lo, p);
                    o[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, pb[q], o[t], 0, 0, 0);
                }
            }
        }
        __syncthreads();
    }
    if (!head_live) return;
    const float inv = sink ? softmax_factor_with_sink(m, l, sink[h0 + col]) : l > 0.f ? 1.0f / l : 0.f;
    float* zr = z + ((size_t)token * H + h0 + col) * R;
#pragma unroll
    for (int t = 0; t < 2 * NS; ++t)
        if (t < 2 * ns) *(f32x4*)(zr + 16 * t + 4 * g) = o[t] * inv;
}

// The same tiles for latents of 128, 256 or 512 values, eight waves to a block.  No wave holds a whole head: for the
// scores of a chunk of 64 keys the waves deal out the keys (four runs of 16) and the steps of 32 values (two halves),
// for the weighted sum the latent's dims, so that every row and every value of a chunk is read from memory by exactly
// one wave of the block, straight into the registers it multiplies from (the values of a chunk are asked for before its
// scores are formed, the rows of the next chunk before this one's are weighted).  What the waves share lies in LDS: the
// folded queries of the tile's 64 (token, head) rows for the whole walk, the halves' scores, and the weights.
//
// Softmax: eight neighbouring threads take a row, eight keys each; a row's maximum and sum live in their registers.
// The base of the exponents follows the maximum lazily, as in the kernel above; where it moved, all waves rescale.
#define LS_S 68               // floats per row of scores (64 and four, so that rows start in different banks)
#define LS_P 72               // values per row of weights
// a barrier that waits for this wave's LDS accesses and not for its loads in flight
__device__ __forceinline__ void lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

template <int NKH, int NDT>
__global__ __launch_bounds__(512, 2) void latent_attention_spread_kernel(
    const bf16_t* __restrict__ qa, float* __restrict__ z, const bf16_t* __restrict__ pool,
    const int* __restrict__ positions, const int* __restrict__ tok_seq, const int* __restrict__ block_table,
    int max_blocks, int H, int K, int R, int page_size, int n_pages, float scale, int window, const int* __restrict__ tiles,
    const float* __restrict__ sink) {
    constexpr int QS = NKH * 64 + 8;
    extern __shared__ __attribute__((aligned(16))) unsigned char lt_smem[];
    bf16_t* qs = (bf16_t*)lt_smem;                                  // [64 rows][QS]
    float* ss = (float*)(qs + 64 * QS);                             // [2 halves][64 rows][LS_S]
    bf16_t* ps = (bf16_t*)(ss + 2 * 64 * LS_S);                     // [64 rows][LS_P]
    float* rs = (float*)(ps + 64 * LS_P);                           // [64 rows]: factor of a chunk, at the end 1 / sum
    int* moved_at = (int*)(rs + 64);                                // the chunk in which some row's base moved last
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
    const int col = lane & 15, g = lane >> 4;
    const int half = wave >> 2, kt = wave & 3;
    const int tile = gridDim.x - 1 - blockIdx.x;                    // (a prompt's last tokens see the most keys: first)
    const int t_first = tiles[4 * tile], n_tok = tiles[4 * tile + 1], g_first = tiles[4 * tile + 2], n_grp = tiles[4 * tile + 3];
    const int nk = K >> 5;
    const int p_max = positions[t_first + n_tok - 1];
    const int* table = block_table + (size_t)tok_seq[t_first] * max_blocks;
    const int lo_min = window > 0 ? max(0, positions[t_first] - window + 1) : 0;
    const size_t page_stride = (size_t)page_size * (K + R);

    // this thread's row in the softmax (and in filling the queries): unit row / 16 = (token, group of 16 heads)
    const int row = tid >> 3, kk = tid & 7;
    const int unit = row >> 4, tw = unit / n_grp, head = (g_first + unit - tw * n_grp) * 16 + (row & 15);
    const bool live = tw < n_tok && head < H;
    const int p = live ? positions[t_first + tw] : -1;
    const int lo = window > 0 ? max(0, p - window + 1) : 0;
    {
        const bf16_t* qr = qa + ((size_t)(t_first + (live ? tw : 0)) * H + (live ? head : 0)) * K;
        const bf16x8 zero = {(bf16_t)0.f, (bf16_t)0.f, (bf16_t)0.f, (bf16_t)0.f, (bf16_t)0.f, (bf16_t)0.f, (bf16_t)0.f, (bf16_t)0.f};
        for (int c = kk; c < NKH * 8; c += 8) {
            const bool inside = live && 8 * c < K;
            const bf16x8 v = *(const bf16x8*)(qr + (inside ? 8 * c : 0));
            *(bf16x8*)(qs + row * QS + 8 * c) = inside ? v : zero;
        }
        if (tid == 0) *moved_at = -1;
    }
    auto page_of = [&](int key) {                                   // (a run beyond the newest token: that token's page, masked below)
        const int page = table[min(key, p_max & ~15) / page_size];
        return pool + (size_t)min(max(page, 0), n_pages - 1) * page_stride;
    };
    bf16x8 kreg[NKH], vreg[NDT][2];
    auto load_keys = [&](int t0) {
        const int key = t0 + 16 * kt;
        const bf16_t* src = page_of(key) + (size_t)(min(key, p_max & ~15) % page_size + col) * K + 8 * g;
#pragma unroll
        for (int i = 0; i < NKH; ++i) {
            const int st = half * NKH + i;
            kreg[i] = *(const bf16x8*)(src + (st < nk ? 32 * st : 0));
        }
    };
    auto load_values = [&](int t0) {
#pragma unroll
        for (int q = 0; q < 2; ++q) {
            const int run = t0 + 32 * q + 16 * (g >> 1);
            const bf16_t* src = page_of(run) + (size_t)page_size * K + min(run, p_max & ~15) % page_size + 8 * (g & 1);
#pragma unroll
            for (int d = 0; d < NDT; ++d) vreg[d][q] = *(const bf16x8*)(src + (size_t)(16 * (NDT * wave + d) + col) * page_size);
        }
    };
    f32x4 o[NDT][4];                                                // dims 16 (NDT wave + d) + 4 g + r of row 16 u + col
#pragma unroll
    for (int d = 0; d < NDT; ++d)
#pragma unroll
        for (int u = 0; u < 4; ++u) o[d][u] = (f32x4){0.f, 0.f, 0.f, 0.f};
    float m = -INFINITY, l = 0.f;
    const int t_begin = lo_min & ~(LT_CHUNK - 1);
    load_keys(t_begin);
    __syncthreads();                                                // the queries are in place
    for (int t0 = t_begin; t0 <= p_max; t0 += LT_CHUNK) {
        load_values(t0);
        f32x4 sacc[4];
#pragma unroll
        for (int u = 0; u < 4; ++u) sacc[u] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < NKH; ++i)
#pragma unroll
            for (int u = 0; u < 4; ++u)
                sacc[u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kreg[i], *(const bf16x8*)(qs + (16 * u + col) * QS + (half * NKH + i) * 32 + 8 * g), sacc[u], 0, 0, 0);
        // lane (row col, g): keys 16 kt + 4 g .. + 3
#pragma unroll
        for (int u = 0; u < 4; ++u) *(f32x4*)(ss + (half * 64 + 16 * u + col) * LS_S + 16 * kt + 4 * g) = sacc[u];
        if (t0 + LT_CHUNK <= p_max) load_keys(t0 + LT_CHUNK);
        lds_barrier();
        {
            float sv[8], cmax = -INFINITY;
#pragma unroll
            for (int h4 = 0; h4 < 2; ++h4) {
                const f32x4 a = *(const f32x4*)(ss + row * LS_S + 8 * kk + 4 * h4), b = *(const f32x4*)(ss + (64 + row) * LS_S + 8 * kk + 4 * h4);
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const int key = t0 + 8 * kk + 4 * h4 + e;
                    sv[4 * h4 + e] = key > p || key < lo ? -INFINITY : (a[e] + b[e]) * scale;
                    cmax = fmaxf(cmax, sv[4 * h4 + e]);
                }
            }
            cmax = fmaxf(cmax, __shfl_xor(cmax, 1, FL_WAVE));
            cmax = fmaxf(cmax, __shfl_xor(cmax, 2, FL_WAVE));
            cmax = fmaxf(cmax, __shfl_xor(cmax, 4, FL_WAVE));
            const float m_new = cmax > m + 8.0f ? cmax : m;         // minus infinity while the row has seen no key
            const float base = m_new == -INFINITY ? 0.f : m_new;
            const float corr = expf(m - base);
            bf16x8 w;
            float lsum = 0.f;
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                w[e] = (bf16_t)expf(sv[e] - base);
                lsum += (float)w[e];                                // the sum of the weights as they are multiplied
            }
            lsum += __shfl_xor(lsum, 1, FL_WAVE);
            lsum += __shfl_xor(lsum, 2, FL_WAVE);
            lsum += __shfl_xor(lsum, 4, FL_WAVE);
            l = l * corr + lsum;
            *(bf16x8*)(ps + row * LS_P + 8 * kk) = w;
            if (kk == 0) rs[row] = corr;
            if (m_new != m) *moved_at = t0;
            m = m_new;
        }
        lds_barrier();
        if (*moved_at == t0) {
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                const float corr = rs[16 * u + col];
#pragma unroll
                for (int d = 0; d < NDT; ++d) o[d][u] *= corr;
            }
        }
        const bool edge = t0 + LT_CHUNK - 1 > p_max || t0 < lo_min;
#pragma unroll
        for (int q = 0; q < 2; ++q) {
            bf16x8 pb[4];
#pragma unroll
            for (int u = 0; u < 4; ++u) pb[u] = *(const bf16x8*)(ps + (16 * u + col) * LS_P + 32 * q + 8 * g);
#pragma unroll
            for (int d = 0; d < NDT; ++d) {
                bf16x8 v = vreg[d][q];
                if (edge) v = keep_keys(v, t0 + 32 * q + 8 * g, lo_min, p_max);          // (what no row of the tile sees is zero, whatever the page holds)
#pragma unroll
                for (int u = 0; u < 4; ++u) o[d][u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, pb[u], o[d][u], 0, 0, 0);
            }
        }
    }
    __syncthreads();
    if (kk == 0) rs[row] = sink && live ? softmax_factor_with_sink(m, l, sink[head]) : l > 0.f ? 1.0f / l : 0.f;
    __syncthreads();
#pragma unroll
    for (int u = 0; u < 4; ++u) {
        const int tu = u / n_grp, hu = (g_first + u - tu * n_grp) * 16 + col;
        if (tu >= n_tok || hu >= H) continue;
        const float inv = rs[16 * u + col];
        float* zr = z + ((size_t)(t_first + tu) * H + hu) * R;
#pragma unroll
        for (int d = 0; d < NDT; ++d) *(f32x4*)(zr + 16 * (NDT * wave + d) + 4 * g) = o[d][u] * inv;
    }
}

template <int NKH, int NDT>
static int launch_spread(const void* qa, float* z, const void* pool, const int* positions, const int* tok_seq, const int* block_table,
                         int max_blocks, int H, int K, int R, int page_size, int n_pages, float scale, int window, const int* tiles,
                         int n_tiles, const float* sink, hipStream_t stream) {
    constexpr int LDS = 64 * (NKH * 64 + 8) * 2 + 2 * 64 * LS_S * 4 + 64 * LS_P * 2 + 64 * 4 + 16;
    static bool sized = false;
    if (!sized) {
        hipError_t e_ = hipFuncSetAttribute((const void*)latent_attention_spread_kernel<NKH, NDT>, hipFuncAttributeMaxDynamicSharedMemorySize, LDS);
        FL_CHECK(e_ == hipSuccess, "latent_attention_spread: %s", hipGetErrorString(e_));
        sized = true;
    }
    latent_attention_spread_kernel<NKH, NDT><<<n_tiles, 512, LDS, stream>>>((const bf16_t*)qa, z, (const bf16_t*)pool, positions, tok_seq, block_table,
                                                                            max_blocks, H, K, R, page_size, n_pages, scale, window, tiles, sink);
    return 0;
}

extern "C" long fl_latent_attention_shared_lds(int K, int R) { return (long)LT_CHUNK * (K + 8) * 2 + (long)R * (LT_CHUNK + 8) * 2; }

// tiles [n_tiles][4] = (first token, tokens, first group of 16 heads, groups): tokens x groups <= 4, the tokens of one request
extern "C" int fl_latent_attention_shared(const void* qa, float* z, const void* pool, const int* positions,
                                          const int* tok_seq, const int* block_table, int max_blocks, int H, int K, int R,
                                          int page_size, int n_pages, float scale, int window, const int* tiles, int n_tiles,
                                          const float* sink, hipStream_t stream) {
    FL_CHECK(n_tiles >= 0 && H > 0 && n_pages > 0 && max_blocks > 0, "latent_attention_shared: bad sizes");
    FL_CHECK(fl_latent_attention_mfma_takes(K, R, page_size), "latent_attention_shared: rows of %d and %d values in pages of %d are not taken", K, R, page_size);
    FL_CHECK((uintptr_t)qa % 16 == 0 && (uintptr_t)pool % 16 == 0 && (uintptr_t)z % 16 == 0, "latent_attention_shared: operands must be 16-byte aligned");
    FL_CHECK(window >= 0, "latent_attention_shared: negative window");
    if (n_tiles == 0) return 0;
    if (R == 128 || R == 256 || R == 512) {
#define FL_LSP(NKH, NDT) launch_spread<NKH, NDT>(qa, z, pool, positions, tok_seq, block_table, max_blocks, H, K, R, page_size, n_pages, scale, window, tiles, n_tiles, sink, stream)
        const int rc = R == 128 ? (K == R ? FL_LSP(2, 1) : FL_LSP(3, 1)) : R == 256 ? (K == R ? FL_LSP(4, 2) : FL_LSP(5, 2)) : K == R ? FL_LSP(8, 4) : FL_LSP(9, 4);
#undef FL_LSP
        if (rc != 0) return rc;
        FL_LAUNCH_CHECK();
        return 0;
    }
    const size_t lds = (size_t)fl_latent_attention_shared_lds(K, R);
    const int ns = R / 32;
#define FL_LTS(NK, NS)                                                                                                     \
    do {                                                                                                               \
        static bool sized = false;                                                                                     \
        if (!sized) {                                                                                                  \
            hipError_t e_ = hipFuncSetAttribute((const void*)latent_attention_shared_kernel<NK, NS>,                      \
                                                hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);              \
            FL_CHECK(e_ == hipSuccess, "latent_attention_shared: %s", hipGetErrorString(e_));                          \
            sized = true;                                                                                              \
        }                                                                                                              \
        latent_attention_shared_kernel<NK, NS><<<n_tiles, 64 * LT_WAVES, lds, stream>>>(                                  \
            (const bf16_t*)qa, z, (const bf16_t*)pool, positions, tok_seq, block_table, max_blocks, H, K, R, page_size,   \
            n_pages, scale, window, tiles, sink);                                                                            \
    } while (0)
    if (K == R) {
        if (ns <= 2) FL_LTS(2, 2);
        else if (ns <= 4) FL_LTS(4, 4);
        else if (ns <= 8) FL_LTS(8, 8);
        else FL_LTS(16, 16);
    } else {
        if (ns <= 2) FL_LTS(4, 2);
        else if (ns <= 4) FL_LTS(6, 4);
        else if (ns <= 8) FL_LTS(10, 8);
        else FL_LTS(18, 16);
    }
#undef FL_LTS
    FL_LAUNCH_CHECK();
    return 0;
}
FL_RECORDABLE(fl_latent_attention_shared)


// The same walk for steps of few rows (decoding), where a wave that holds all of a latent's dims has no register
// left for reads in flight and waits for every operand: the four waves of a block take one (token, 16 heads, part
// of the keys) together and deal the latent's steps of 32 dims out among them (wave w: steps w, w + 4, ...).
// Each forms its share of the scores, the shares are added through LDS in a fixed order (every wave gets the
// same sums, hence the same maxima and weights), and each adds the weighted rows of its own dims.  A wave then
// holds a quarter of the accumulators and queries, and the reads of a chunk are all in flight at once.
template <int NKW, int NSW>
__global__ __launch_bounds__(64 * LT_WAVES) void latent_attention_dealt_kernel(
    const bf16_t* __restrict__ qa, float* __restrict__ z, const bf16_t* __restrict__ pool,
    const int* __restrict__ positions, const int* __restrict__ tok_seq, const int* __restrict__ block_table,
    int max_blocks, int n, int H, int K, int R, int page_size, int n_pages, float scale, int window, int groups_per_token,
    int n_split, float* __restrict__ part_o, float* __restrict__ part_ml, const float* __restrict__ sink) {
    __shared__ f32x4 sx[LT_WAVES][4][64];
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int unit = blockIdx.x;                                   // (token, group of 16 heads, part of the keys)
    const int split = unit % n_split, tg = unit / n_split;
    const int token = tg / groups_per_token, h0 = (tg - token * groups_per_token) * 16;
    const int col = lane & 15, g = lane >> 4;
    const int nk = K >> 5, ns = R >> 5;
    const int p = positions[token];
    const int* table = block_table + (size_t)tok_seq[token] * max_blocks;
    const int lo = window > 0 ? max(0, p - window + 1) : 0;
    const size_t page_stride = (size_t)page_size * (K + R);
    const bool head_live = h0 + col < H;
    bf16x8 qreg[NKW];
    {
        const bf16_t* qr = qa + ((size_t)token * H + h0 + (head_live ? col : 0)) * K;
#pragma unroll
        for (int i = 0; i < NKW; ++i) {
            const int s = wave + LT_WAVES * i;
            if (s < nk && head_live) {
                qreg[i] = *(const bf16x8*)(qr + 32 * s + 8 * g);
            } else {
#pragma unroll
                for (int e = 0; e < 8; ++e) qreg[i][e] = (bf16_t)0.f;
            }
        }
    }
    f32x4 o[2 * NSW];                                              // dims 32 s + 16 u + 4 g + r of the wave's steps s, u = 0, 1
#pragma unroll
    for (int t = 0; t < 2 * NSW; ++t) o[t] = (f32x4){0.f, 0.f, 0.f, 0.f};
    float m = -INFINITY, l = 0.f;
    int first = lo & ~(LT_CHUNK - 1), last = p;
    if (n_split > 1) {
        const int chunks = (p - first) / LT_CHUNK + 1, per = (chunks + n_split - 1) / n_split;
        last = min(p, first + (split + 1) * per * LT_CHUNK - 1);
        first += split * per * LT_CHUNK;
    }
    for (int t0 = first; t0 <= last; t0 += LT_CHUNK) {
        // the values do not wait for the scores: all of a chunk's reads are asked for at its start
        int key0[2];
        bf16x8 vreg[2 * NSW][2];
#pragma unroll
        for (int q = 0; q < 2; ++q) {
            key0[q] = t0 + 32 * q + 8 * g;
            const int kc = min(key0[q], p);
            int page = table[kc / page_size];
            page = min(max(page, 0), n_pages - 1);
            const bf16_t* cols = pool + (size_t)page * page_stride + (size_t)page_size * K + (key0[q] % page_size);
#pragma unroll
            for (int t = 0; t < 2 * NSW; ++t) {
                const int s = wave + LT_WAVES * (t >> 1);
                vreg[t][q] = *(const bf16x8*)(cols + (size_t)((s < ns ? 32 * s : 0) + 16 * (t & 1) + col) * page_size);
            }
        }
        f32x4 sacc[4];
#pragma unroll
        for (int a = 0; a < 4; ++a) {
            sacc[a] = (f32x4){0.f, 0.f, 0.f, 0.f};
            const int key = t0 + 32 * (a >> 1) + 8 * (col >> 2) + 4 * (a & 1) + (col & 3);
            const int kc = min(key, p);
            int page = table[kc / page_size];
            page = min(max(page, 0), n_pages - 1);
            const bf16_t* row = pool + (size_t)page * page_stride + (size_t)(kc % page_size) * K + 8 * g;
#pragma unroll
            for (int i = 0; i < NKW; ++i) {
                const int s = wave + LT_WAVES * i;
                sacc[a] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*(const bf16x8*)(row + (s < nk ? 32 * s : 0)), qreg[i], sacc[a], 0, 0, 0);
            }
            sx[wave][a][lane] = sacc[a];
        }
        __syncthreads();
        float cmax = -INFINITY;
#pragma unroll
        for (int a = 0; a < 4; ++a) {
            sacc[a] = (sx[0][a][lane] + sx[1][a][lane]) + (sx[2][a][lane] + sx[3][a][lane]);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int key = t0 + 32 * (a >> 1) + 8 * g + 4 * (a & 1) + e;
                sacc[a][e] = key > p || key < lo ? -INFINITY : sacc[a][e] * scale;
                cmax = fmaxf(cmax, sacc[a][e]);
            }
        }
        __syncthreads();                                           // (the next chunk's shares overwrite sx)
        cmax = fmaxf(cmax, __shfl_xor(cmax, 16, FL_WAVE));
        cmax = fmaxf(cmax, __shfl_xor(cmax, 32, FL_WAVE));
        const float m_new = fmaxf(m, cmax);
        const float corr = expf(m - m_new);
        m = m_new;
        bf16x8 pb[2];
        float lsum = 0.f;
#pragma unroll
        for (int a = 0; a < 4; ++a)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const bf16_t w = (bf16_t)expf(sacc[a][e] - m_new);
                pb[a >> 1][4 * (a & 1) + e] = w;
                lsum += (float)w;
            }
        lsum += __shfl_xor(lsum, 16, FL_WAVE);
        lsum += __shfl_xor(lsum, 32, FL_WAVE);
        l = l * corr + lsum;
        const bool edge = t0 + LT_CHUNK - 1 > p || t0 < lo;
#pragma unroll
        for (int t = 0; t < 2 * NSW; ++t) {
            o[t] *= corr;
#pragma unroll
            for (int q = 0; q < 2; ++q) {
                bf16x8 v = vreg[t][q];
                if (edge) v = keep_keys(v, key0[q], lo, p);
                o[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, pb[q], o[t], 0, 0, 0);
            }
        }
    }
    if (n_split > 1) {
        float* po = part_o + ((size_t)unit * 16 + col) * R;
#pragma unroll
        for (int t = 0; t < 2 * NSW; ++t) {
            const int s = wave + LT_WAVES * (t >> 1);
            if (s < ns) *(f32x4*)(po + 32 * s + 16 * (t & 1) + 4 * g) = o[t];
        }
        if (wave == 0 && g == 0) {
            part_ml[((size_t)unit * 16 + col) * 2] = m;
            part_ml[((size_t)unit * 16 + col) * 2 + 1] = l;
        }
        return;
    }
    if (!head_live) return;
    const float inv = sink ? softmax_factor_with_sink(m, l, sink[h0 + col]) : l > 0.f ? 1.0f / l : 0.f;
    float* zr = z + ((size_t)token * H + h0 + col) * R;
#pragma unroll
    for (int t = 0; t < 2 * NSW; ++t) {
        const int s = wave + LT_WAVES * (t >> 1);
        if (s < ns) *(f32x4*)(zr + 32 * s + 16 * (t & 1) + 4 * g) = o[t] * inv;
    }
}

// fl_latent_attention_mfma with a block of four waves per (token, 16 heads, part of the keys): for steps of few rows
extern "C" int fl_latent_attention_dealt(const void* qa, float* z, const void* pool, const int* positions,
                                         const int* tok_seq, const int* block_table, int max_blocks, int n, int H, int K, int R,
                                         int page_size, int n_pages, float scale, int window, int n_split, float* part_o,
                                         float* part_ml, const float* sink, hipStream_t stream) {
    FL_CHECK(n >= 0 && H > 0 && n_pages > 0 && max_blocks > 0, "latent_attention_dealt: bad sizes");
    FL_CHECK(n_split >= 1 && n_split <= 64 && (n_split == 1 || (part_o && part_ml)), "latent_attention_dealt: %d parts of the keys (at most 64) need a workspace", n_split);
    FL_CHECK(fl_latent_attention_mfma_takes(K, R, page_size), "latent_attention_dealt: rows of %d and %d values in pages of %d are not taken", K, R, page_size);
    FL_CHECK((uintptr_t)qa % 16 == 0 && (uintptr_t)pool % 16 == 0 && (uintptr_t)z % 16 == 0, "latent_attention_dealt: operands must be 16-byte aligned");
    FL_CHECK(window >= 0, "latent_attention_dealt: negative window");
    if (n == 0) return 0;
    const int groups = ceil_div(H, 16);
    const long units = (long)n * groups * n_split;
    FL_CHECK(units < (1L << 30), "latent_attention_dealt: too many rows");
    const int nkw = ceil_div(K / 32, LT_WAVES), nsw = ceil_div(R / 32, LT_WAVES);
#define FL_LTD(NKW, NSW)                                                                                                       \
    latent_attention_dealt_kernel<NKW, NSW><<<(unsigned)units, 64 * LT_WAVES, 0, stream>>>((const bf16_t*)qa, z, (const bf16_t*)pool, \
                                                                                      positions, tok_seq, block_table, max_blocks, \
                                                                                      n, H, K, R, page_size, n_pages, scale, window,  \
                                                                                      groups, n_split, part_o, part_ml, sink)
    if (nkw <= 1) FL_LTD(1, 1);
    else if (nkw <= 2) FL_LTD(2, 2);
    else if (nsw <= 2 && nkw <= 3) FL_LTD(3, 2);
    else if (nkw <= 4) FL_LTD(4, 4);
    else FL_LTD(5, 4);
#undef FL_LTD
    FL_LAUNCH_CHECK();
    if (n_split > 1) {
        dim3 mgrid(n * H, ceil_div(R, 256));
        latent_merge_kernel<<<mgrid, 256, 0, stream>>>(part_o, part_ml, z, H, R, groups, n_split, sink);
        FL_LAUNCH_CHECK();
    }
    return 0;
}
FL_RECORDABLE(fl_latent_attention_dealt)

// ------------------------------------------------------------------ one product per head on the matrix cores
// out[t][h][j] = sum_k x[t][h][k] w[h][j][k]   (x float or bfloat16 rows ldx apart, head h at h * hx; w bfloat16
// [H][J][K], K a multiple of 8, J of 16; heads ho apart in out), optionally times sigmoid(gate[t][gate_col0 + h]); tail:
// what stands behind a head's J results (query_tail.h).  A wave takes 16 tokens of one head: its x is
// the B operand, held in registers for all of K; the weights are the A operand, so a lane ends with four
// consecutive outputs of one token.
template <typename TX, typename TOut, int NS>
__global__ __launch_bounds__(64 * LT_WAVES) void heads_matmul_mfma_kernel(
    const TX* __restrict__ x, int ldx, int hx, const bf16_t* __restrict__ w, TOut* __restrict__ out, int ho, int n, int H, int K, int J,
    const float* __restrict__ gate, int ldg, int gate_col0, int j_parts, QueryTail tail) {
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    // a wave takes 16 tokens and every j_parts-th tile of 16 output columns (few tokens: many parts, so that
    // a decode step still fills the chip)
    const int unit = blockIdx.x * LT_WAVES + wave;
    const int t0 = (unit / j_parts) * 16, j_first = unit % j_parts, h = blockIdx.y;
    if (t0 >= n) return;
    const int col = lane & 15, g = lane >> 4;
    const int token = t0 + col;
    const bool live = token < n;
    bf16x8 xreg[NS];
    {
        const TX* xr = x + (size_t)(live ? token : t0) * ldx + (size_t)h * hx;
#pragma unroll
        for (int s = 0; s < NS; ++s) {
            const bool inside = 32 * s + 8 * g < K;
            const TX* src = xr + (inside ? 32 * s + 8 * g : 0);        // (no branch around a load: what lies beyond K or n is set to zero afterwards)
            TX v[8];
#pragma unroll
            for (int e = 0; e < 8; ++e) v[e] = src[e];
#pragma unroll
            for (int e = 0; e < 8; ++e) xreg[s][e] = inside && live ? (bf16_t)to_f32(v[e]) : (bf16_t)0.f;
        }
    }
    const float gv = (gate && live) ? 1.0f / (1.0f + expf(-gate[(size_t)token * ldg + gate_col0 + h])) : 1.0f;
    const bf16_t* wh = w + (size_t)h * J * K;
#pragma unroll 4
    for (int jt = j_first; jt < J / 16; jt += j_parts) {
        f32x4 acc = (f32x4){0.f, 0.f, 0.f, 0.f};
        const bf16_t* row = wh + (size_t)(16 * jt + col) * K + 8 * g;
#pragma unroll
        for (int s = 0; s < NS; ++s)
            acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*(const bf16x8*)(32 * s + 8 * g < K ? row + 32 * s : row - 8 * g), xreg[s], acc, 0, 0, 0);      // (beyond K: finite weights against zeros)
        if (live) {
            TOut* dst = out + ((size_t)token * H + h) * ho + 16 * jt + 4 * g;
#pragma unroll
            for (int r = 0; r < 4; ++r) dst[r] = from_f32<TOut>(acc[r] * gv);
        }
    }
    if constexpr (std::is_same<TX, float>::value) {
        if (tail.width > 0 && j_first == 0)
            for (int e = lane; e < 16 * tail.width; e += 64) {
                const int i = e / tail.width, d = e - i * tail.width;
                if (t0 + i < n)
                    out[((size_t)(t0 + i) * H + h) * ho + J + d] =
                        from_f32<TOut>(query_tail_value(tail, x + (size_t)(t0 + i) * ldx + (size_t)h * hx, t0 + i, d));
            }
    }
}

extern "C" int fl_heads_matmul_mfma_takes(int K, int J) { return K > 0 && K % 8 == 0 && K <= 512 && J > 0 && J % 16 == 0; }

extern "C" int fl_heads_matmul_mfma(const void* x, int x_dtype, int ldx, int hx, const void* w, void* out, int out_dtype, int ho,
                                    int n, int H, int K, int J, const float* gate, int ldg, int gate_col0, int rot_dim, int rot,
                                    int interleaved, const float* cs, int rot_at, hipStream_t stream) {
    FL_CHECK(n >= 0 && H > 0 && hx >= K + rot_dim && ho >= J && (long)ldx >= (long)(H - 1) * hx + K + rot_dim, "heads_matmul_mfma: bad sizes");
    FL_CHECK(rot_dim >= 0 && rot >= 0 && rot % 2 == 0 && rot <= rot_dim && (rot == 0 || cs) && (rot_dim == 0 || (rot_at >= J && rot_at + rot_dim <= ho)),
             "heads_matmul_mfma: a rotated part of %d (%d turned) at %d of %d", rot_dim, rot, rot_at, ho);
    FL_CHECK(ho == J || x_dtype == FL_F32, "heads_matmul_mfma: what stands behind a head's results is made of float rows");
    const QueryTail tail = {ho - J, K, rot_at - J, rot_dim, rot, interleaved, cs};
    FL_CHECK(fl_heads_matmul_mfma_takes(K, J), "heads_matmul_mfma: %d x %d per head is not taken", J, K);
    FL_CHECK((uintptr_t)w % 16 == 0, "heads_matmul_mfma: the weights must be 16-byte aligned");
    FL_CHECK(!gate || ldg >= gate_col0 + H, "heads_matmul_mfma: gate columns beyond rows %d wide", ldg);
    if (n == 0) return 0;
    FL_CHECK(H <= 65535, "heads_matmul_mfma: too many heads");
    // enough waves for four per compute unit, as far as the column tiles go
    const int groups = ceil_div(n, 16);
    int j_parts = (4 * fl_units()) / (groups * H);
    j_parts = j_parts < 1 ? 1 : (j_parts > J / 16 ? J / 16 : j_parts);
    dim3 grid(ceil_div(groups * j_parts, LT_WAVES), H);
    const int ns = (K + 31) / 32;
#define FL_HMM(TX, TO, NS) heads_matmul_mfma_kernel<TX, TO, NS><<<grid, 64 * LT_WAVES, 0, stream>>>((const TX*)x, ldx, hx, (const bf16_t*)w, (TO*)out, ho, n, H, K, J, gate, ldg, gate_col0, j_parts, tail)
#define FL_HMM_NS(TX, TO)                      \
    do {                                       \
        if (ns <= 2) FL_HMM(TX, TO, 2);        \
        else if (ns <= 4) FL_HMM(TX, TO, 4);   \
        else if (ns <= 8) FL_HMM(TX, TO, 8);   \
        else FL_HMM(TX, TO, 16);               \
    } while (0)
    if (x_dtype == FL_F32 && out_dtype == FL_BF16) FL_HMM_NS(float, bf16_t);
    else if (x_dtype == FL_F32 && out_dtype == FL_F32) FL_HMM_NS(float, float);
    else if (x_dtype == FL_BF16 && out_dtype == FL_BF16) FL_HMM_NS(bf16_t, bf16_t);
    else FL_CHECK(false, "heads_matmul_mfma: unsupported dtypes x=%d out=%d", x_dtype, out_dtype);
#undef FL_HMM_NS
#undef FL_HMM
    FL_LAUNCH_CHECK();
    return 0;
}
FL_RECORDABLE(fl_heads_matmul_mfma)
