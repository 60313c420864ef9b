// Attention over one cached latent per token.
//
// A token keeps one normed row c [R] in the paged cache; every head's keys and values are linear in c
// (k = Wk_h c, v = Wv_h c), so the key expansion is folded into the query and the value expansion is
// applied after the weighted sum:
//     qa_h = Wk_h^T q_h                      (fl_heads_matmul, weights as they are)
//     s_j  = scale * qa_h . c_j,  p = softmax over the visible j
//     z_h  = sum_j p_j c_j                    (fl_latent_attention)
//     o_h  = sigmoid(gate_h) * Wv_h z_h       (fl_heads_matmul, weights transposed, gated)
// A row may hold more than the latent: one key part r [rot_dim], rotated by position and shared by the heads,
// behind it.  A head's folded query then carries its own rotated part behind qa_h, the score is their product
// over the whole row, and only the latent is summed.  A row is K values wide as a key and V as a value, both
// rounded up with zeros to what the kernels want: [c | zeros to V | r | zeros to K].
// Scores, softmax, z and the two small products are 32-bit whatever the storage type of the cache.
#include "common.h"
#include "api.h"
#include "recordable.h"
#include "query_tail.h"

// ------------------------------------------------------------------ from the low projections to the latents
// x: float rows ld wide, the joined projection of a step's tokens.  Two blocks per token: one norms the query
// latent, out[r, :] = v * w * rsqrt(mean(v^2) + eps), v = x[r, 0 : q_width]; the other norms the cached latent (the
// columns kv_col .. kv_col + R - 1) and stores it in the page row of the token's position, and turns the rot_dim
// columns behind it by the token's angles (cs [n][rot / 2][2]; dimension i with i + rot / 2 or, interleaved, 2i with
// 2i + 1, those from rot on as they are) into the row's tail.  A page holds [page_size][K] rows and, behind them, [V][page_size] transposed
// values; the matrix cores want the index that is summed over contiguous, a row's values for the scores and the keys
// for the weighted sum.
template <typename T>
__global__ __launch_bounds__(256) void latent_prepare_kernel(
    const float* __restrict__ x, int ld, int q_width, const float* __restrict__ qw, T* __restrict__ q_out, int kv_col,
    int R, const float* __restrict__ kw, float eps, int rot_dim, int rot, int interleaved, const float* __restrict__ cs,
    T* __restrict__ pool, int K, int V, const int* __restrict__ positions, const int* __restrict__ tok_seq,
    const int* __restrict__ block_table, int max_blocks, int page_size, int n_pages) {
    __shared__ float red[4];
    const int r = blockIdx.x;
    const bool query = blockIdx.y == 0;
    const int width = query ? q_width : R;
    const float* xr = x + (size_t)r * ld + (query ? 0 : kv_col);
    const float* w = query ? qw : kw;
    float ss = 0.f;
    for (int i = threadIdx.x; i < width; i += 256) ss += xr[i] * xr[i];
    const float total = block_sum<4>(ss, red);
    const float inv = 1.0f / sqrtf(total / (float)width + eps);
    if (query) {
        T* dst = q_out + (size_t)r * width;
        for (int i = threadIdx.x; i < width; i += 256) dst[i] = from_f32<T>(xr[i] * (w ? w[i] : 1.0f) * inv);
        return;
    }
    const int pos = positions[r];
    const int page = block_table[(size_t)tok_seq[r] * max_blocks + pos / page_size];
    if (page < 0 || page >= n_pages) return;          // rows that pad a batch of fixed shape
    const int row = pos % page_size;
    T* rows = pool + (size_t)page * page_size * (K + V);
    T* cols = rows + (size_t)page_size * K;
    const float* xt = xr + R;
    for (int i = threadIdx.x; i < K; i += 256) {
        float v = 0.f;
        if (i < R) v = xr[i] * (w ? w[i] : 1.0f) * inv;
        else if (i >= V && i < V + rot_dim) v = rotated_value(xt, i - V, rot, interleaved, cs + (size_t)r * rot);
        rows[(size_t)row * K + i] = from_f32<T>(v);
        if (i < V) cols[(size_t)i * page_size + row] = from_f32<T>(v);
    }
}

extern "C" int fl_latent_prepare(const float* x, int ld, int q_width, const float* qw, void* q_out, int kv_col, int R,
                                 const float* kw, float eps, int rot_dim, int rot, int interleaved, const float* cs, void* pool, int dtype,
                                 int K, int V, int n, const int* positions, const int* tok_seq, const int* block_table,
                                 int max_blocks, int page_size, int n_pages, int write_cache, hipStream_t stream) {
    FL_CHECK(n >= 0 && q_width > 0 && R > 0 && kv_col >= 0 && rot_dim >= 0 && ld >= q_width && ld >= kv_col + R + rot_dim,
             "latent_prepare: columns 0..%d and %d..%d of rows %d wide", q_width, kv_col, kv_col + R + rot_dim, ld);
    FL_CHECK(V >= R && K >= V + rot_dim, "latent_prepare: a latent of %d and a rotated part of %d in rows of %d, values of %d", R, rot_dim, K, V);
    FL_CHECK(rot >= 0 && rot % 2 == 0 && rot <= rot_dim && (rot == 0 || cs), "latent_prepare: %d rotated dims of %d, or no table", rot, rot_dim);
    FL_CHECK(!write_cache || (pool && positions && tok_seq && block_table && max_blocks > 0 && page_size > 0 && n_pages > 0), "latent_prepare: a paged store needs positions, requests and the pool's sizes");
    if (n == 0) return 0;
    dim3 grid(n, write_cache ? 2 : 1);
    if (dtype == FL_F32)
        latent_prepare_kernel<float><<<grid, 256, 0, stream>>>(x, ld, q_width, qw, (float*)q_out, kv_col, R, kw, eps, rot_dim, rot, interleaved, cs, (float*)pool, K, V, positions, tok_seq, block_table, max_blocks, page_size, n_pages);
    else if (dtype == FL_BF16)
        latent_prepare_kernel<bf16_t><<<grid, 256, 0, stream>>>(x, ld, q_width, qw, (bf16_t*)q_out, kv_col, R, kw, eps, rot_dim, rot, interleaved, cs, (bf16_t*)pool, K, V, positions, tok_seq, block_table, max_blocks, page_size, n_pages);
    else
        FL_CHECK(false, "latent_prepare: unknown dtype %d", dtype);
    FL_LAUNCH_CHECK();
    return 0;
}
FL_RECORDABLE(fl_latent_prepare)

// ------------------------------------------------------------------ one small product per head
// x: float rows ldx apart, head h's K values at h * hx; one matrix per head taken from w [H * rows_per_head][cols]:
//   transposed = 0: w_h is [K][J] (rows_per_head = K, cols = J),   out[t][h][j] = sum_k x[t][h][k] w_h[k][j]
//   transposed = 1: w_h is [J][K] (rows_per_head = J, cols = K),   out[t][h][j] = sum_k x[t][h][k] w_h[j][k]
// Head h's results lie ho apart in out (ho >= J).  tail: what stands behind a head's J results (query_tail.h).
// gate (or null): float rows ldg apart, gate[t][gate_col0 + h] is a logit; the head's output is multiplied
// by its sigmoid.  A block takes HM_TOKENS tokens of one head; a thread owns output columns and keeps
// one sum per token, so every weight is read once per block.  Sums run over k in rising order.
#define HM_TOKENS 8
template <typename TW, typename TOut>
__global__ __launch_bounds__(256) void heads_matmul_kernel(const float* __restrict__ x, int ldx, const TW* __restrict__ w,
                                                           int hx, TOut* __restrict__ out, int ho, int n, int H, int K,
                                                           int J, int transposed, const float* __restrict__ gate, int ldg,
                                                           int gate_col0, QueryTail tail) {
    extern __shared__ float xs[];                     // [HM_TOKENS][K]
    const int t0 = blockIdx.x * HM_TOKENS, h = blockIdx.y;
    const int nt = min(HM_TOKENS, n - t0);
    for (int e = threadIdx.x; e < HM_TOKENS * K; e += 256) {
        const int i = e / K, k = e - i * K;
        xs[e] = i < nt ? x[(size_t)(t0 + i) * ldx + (size_t)h * hx + k] : 0.f;
    }
    __syncthreads();
    const TW* wh = w + (size_t)h * K * J;             // either form holds K * J values per head
    for (int j = threadIdx.x; j < J; j += 256) {
        float acc[HM_TOKENS];
#pragma unroll
        for (int i = 0; i < HM_TOKENS; ++i) acc[i] = 0.f;
        if (transposed) {
            const TW* row = wh + (size_t)j * K;
            for (int k = 0; k < K; ++k) {
                const float wv = to_f32(row[k]);
#pragma unroll
                for (int i = 0; i < HM_TOKENS; ++i) acc[i] = fmaf(xs[i * K + k], wv, acc[i]);
            }
        } else {
            for (int k = 0; k < K; ++k) {
                const float wv = to_f32(wh[(size_t)k * J + j]);
#pragma unroll
                for (int i = 0; i < HM_TOKENS; ++i) acc[i] = fmaf(xs[i * K + k], wv, acc[i]);
            }
        }
#pragma unroll
        for (int i = 0; i < HM_TOKENS; ++i) {
            if (i >= nt) break;
            float v = acc[i];
            if (gate) v *= 1.0f / (1.0f + expf(-gate[(size_t)(t0 + i) * ldg + gate_col0 + h]));
            out[((size_t)(t0 + i) * H + h) * ho + j] = from_f32<TOut>(v);
        }
    }
    if (tail.width > 0)
        for (int e = threadIdx.x; e < nt * tail.width; e += 256) {
            const int i = e / tail.width, d = e - i * tail.width;
            out[((size_t)(t0 + i) * H + h) * ho + J + d] =
                from_f32<TOut>(query_tail_value(tail, x + (size_t)(t0 + i) * ldx + (size_t)h * hx, t0 + i, d));
        }
}

extern "C" int fl_heads_matmul(const float* x, int ldx, int hx, const void* w, int w_dtype, void* out, int out_dtype, int ho,
                               int n, int H, int K, int J, int transposed, const float* gate, int ldg, int gate_col0,
                               int rot_dim, int rot, int interleaved, const float* cs, int rot_at, hipStream_t stream) {
    FL_CHECK(n >= 0 && H > 0 && K > 0 && J > 0 && hx >= K + rot_dim && ho >= J && (long)ldx >= (long)(H - 1) * hx + K + rot_dim,
             "heads_matmul: bad sizes n=%d H=%d K=%d J=%d ld=%d head strides %d, %d", n, H, K, J, ldx, hx, ho);
    FL_CHECK(rot_dim >= 0 && rot >= 0 && rot % 2 == 0 && rot <= rot_dim && (rot == 0 || cs) && (rot_dim == 0 || (rot_at >= J && rot_at + rot_dim <= ho)),
             "heads_matmul: a rotated part of %d (%d turned) at %d of %d", rot_dim, rot, rot_at, ho);
    const QueryTail tail = {ho - J, K, rot_at - J, rot_dim, rot, interleaved, cs};
    const size_t lds = (size_t)HM_TOKENS * K * sizeof(float);
    FL_CHECK(lds <= 64 * 1024, "heads_matmul: %d values per head are more than a block keeps", K);
    FL_CHECK(!gate || ldg >= gate_col0 + H, "heads_matmul: gate columns %d..%d of rows %d wide", gate_col0, gate_col0 + H, ldg);
    if (n == 0) return 0;
    dim3 grid(ceil_div(n, HM_TOKENS), H);
#define FL_HM(TW, TO) heads_matmul_kernel<TW, TO><<<grid, 256, lds, stream>>>(x, ldx, (const TW*)w, hx, (TO*)out, ho, n, H, K, J, transposed, gate, ldg, gate_col0, tail)
    if (w_dtype == FL_F32 && out_dtype == FL_F32) FL_HM(float, float);
    else if (w_dtype == FL_BF16 && out_dtype == FL_F32) FL_HM(bf16_t, float);
    else if (w_dtype == FL_BF16 && out_dtype == FL_BF16) FL_HM(bf16_t, bf16_t);
    else FL_CHECK(false, "heads_matmul: unsupported dtypes w=%d out=%d", w_dtype, out_dtype);
#undef FL_HM
    FL_LAUNCH_CHECK();
    return 0;
}
FL_RECORDABLE(fl_heads_matmul)

// ------------------------------------------------------------------ attention over the latent rows
// One block per (token, group of heads); a wave takes LA_HPW heads one after the other.  Keys come in
// chunks of 64: a lane scores one key against the head's folded query (kept in LDS), the wave takes
// maximum and sum, then lanes own the latent's dims (R: a row's values, the first of its K) and add the chunk's weighted rows.  The query at
// position p sees keys 0..p of its own request (window > 0: the newest `window` of them), all read
// from the pages (this step's rows were stored before).  Rows beyond p are never loaded, so whatever
// an unused or reused page holds cannot reach a sum.  sink (float [H], or null): a score per head that joins the
// denominator once, not scaled, with no key and no value.
#define LA_WAVES 4
#define LA_MAX_DIMS 16        // latent dims per lane: R <= 64 * LA_MAX_DIMS
template <typename T, int VPL>
__global__ __launch_bounds__(64 * LA_WAVES) void latent_attention_kernel(
    const float* __restrict__ qa, float* __restrict__ z, const T* __restrict__ pool, const int* __restrict__ positions,
    const int* __restrict__ tok_seq, const int* __restrict__ block_table, int max_blocks, int H, int K, int R, int page_size,
    int n_pages, float scale, int window, int heads_per_block, const float* __restrict__ sink) {
    extern __shared__ float lds[];                    // [heads_per_block][K] folded queries, then [LA_WAVES][64] weights
    const int token = blockIdx.x;
    const int h0 = blockIdx.y * heads_per_block;
    const int nh = min(heads_per_block, H - h0);
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    float* qs = lds;
    volatile float* ps = lds + (size_t)heads_per_block * K + wave * 64;   // written and read by this wave alone
    for (int e = threadIdx.x; e < nh * K; e += 64 * LA_WAVES) qs[e] = qa[((size_t)token * H + h0) * K + e] * scale;
    const size_t page_stride = (size_t)page_size * (K + R);
    __syncthreads();
    const int p = positions[token];
    const int* table = block_table + (size_t)tok_seq[token] * max_blocks;
    const int lo = window > 0 ? max(0, p - window + 1) : 0;
    for (int hh = wave; hh < nh; hh += LA_WAVES) {
        const float* qh = qs + (size_t)hh * K;
        float acc[VPL];
#pragma unroll
        for (int u = 0; u < VPL; ++u) acc[u] = 0.f;
        float m = -INFINITY, l = 0.f;
        for (int t0 = lo; t0 <= p; t0 += 64) {
            const int t = t0 + lane;
            float s = -INFINITY;
            if (t <= p) {
                const int page = table[t / page_size];
                const T* row = pool + (size_t)page * page_stride + (size_t)(t % page_size) * K;
                float a = 0.f;
                if (page >= 0 && page < n_pages)
                    for (int d = 0; d < K; ++d) a = fmaf(qh[d], to_f32(row[d]), a);
                s = a;
            }
            const float m_new = fmaxf(m, wave_max(s));
            const float corr = expf(m - m_new);       // 0 in the first chunk
            const float e = t <= p ? expf(s - m_new) : 0.f;
            l = l * corr + wave_sum(e);
            m = m_new;
            ps[lane] = e;
            __builtin_amdgcn_wave_barrier();
            const int cnt = min(64, p - t0 + 1);
#pragma unroll
            for (int u = 0; u < VPL; ++u) acc[u] *= corr;
            for (int j = 0; j < cnt; ++j) {
                const int tj = t0 + j;
                const int page = table[tj / page_size];
                if (page < 0 || page >= n_pages) continue;          // (rows that pad a batch of fixed shape have no pages)
                const T* row = pool + (size_t)page * page_stride + (size_t)(tj % page_size) * K;
                const float w = ps[j];
#pragma unroll
                for (int u = 0; u < VPL; ++u) {
                    const int d = lane + 64 * u;
                    if (d < R) acc[u] = fmaf(w, to_f32(row[d]), acc[u]);
                }
            }
            __builtin_amdgcn_wave_barrier();
        }
        const float inv = sink ? softmax_factor_with_sink(m, l, sink[h0 + hh]) : l > 0.f ? 1.0f / l : 0.f;
        float* zr = z + ((size_t)token * H + h0 + hh) * R;
#pragma unroll
        for (int u = 0; u < VPL; ++u) {
            const int d = lane + 64 * u;
            if (d < R) zr[d] = acc[u] * inv;
        }
    }
}

extern "C" int fl_latent_max_width(void) { return 64 * LA_MAX_DIMS; }

extern "C" int fl_latent_attention(const float* qa, float* z, const void* pool, int dtype, const int* positions,
                                   const int* tok_seq, const int* block_table, int max_blocks, int n, int H, int K, int R,
                                   int page_size, int n_pages, float scale, int window, const float* sink, hipStream_t stream) {
    FL_CHECK(n >= 0 && H > 0 && R > 0 && K >= R && K <= 2 * 64 * LA_MAX_DIMS && page_size > 0 && n_pages > 0 && max_blocks > 0, "latent_attention: bad sizes");
    FL_CHECK(R <= 64 * LA_MAX_DIMS, "latent_attention: a latent of %d values, at most %d", R, 64 * LA_MAX_DIMS);
    FL_CHECK(window >= 0, "latent_attention: negative window");
    if (n == 0) return 0;
    // as many heads per block as keep the folded queries within 32 KB; a wave walks its heads in turn
    int hpb = (int)((32 * 1024) / ((size_t)R * sizeof(float)));
    hpb = hpb < 1 ? 1 : (hpb > H ? H : hpb);
    if (hpb > 2 * LA_WAVES) hpb = 2 * LA_WAVES;
    const size_t lds = ((size_t)hpb * K + 64 * LA_WAVES) * sizeof(float);
    dim3 grid(n, ceil_div(H, hpb));
    const int vpl = ceil_div(R, 64);
#define FL_LA(TT, V)                                                                                                  \
    latent_attention_kernel<TT, V><<<grid, 64 * LA_WAVES, lds, stream>>>(qa, z, (const TT*)pool, positions, tok_seq, \
                                                                         block_table, max_blocks, H, K, R, page_size, \
                                                                         n_pages, scale, window, hpb, sink)
#define FL_LA_V(TT)                                  \
    do {                                             \
        if (vpl <= 1) FL_LA(TT, 1);                  \
        else if (vpl <= 2) FL_LA(TT, 2);             \
        else if (vpl <= 4) FL_LA(TT, 4);             \
        else if (vpl <= 8) FL_LA(TT, 8);             \
        else FL_LA(TT, LA_MAX_DIMS);                 \
    } while (0)
    if (dtype == FL_F32) FL_LA_V(float);
    else if (dtype == FL_BF16) FL_LA_V(bf16_t);
    else FL_CHECK(false, "latent_attention: unknown dtype %d", dtype);
#undef FL_LA_V
#undef FL_LA
    FL_LAUNCH_CHECK();
    return 0;
}
FL_RECORDABLE(fl_latent_attention)
