// What stands around a sublayer that is normed on both sides: the way of its output into the residual stream, and the
// short convolution over time in front of its mixer.
//
//   fl_sublayer_step   resid += scale * norm(sigmoid(gate + gate_bias) * y), and optionally the norm of the new
//                      stream, which the next sublayer reads.  Gate and scale are optional; either norm is a layer norm
//                      (mean and variance) or a root-mean-square norm, with eps inside the root.  y may arrive as the
//                      rows of a token's experts, which are added here in rising rank.
//   fl_input_conv      out_t = h_t + sum_k w_k h_(t - taps + 1 + k) per channel, zeros before a sequence's start
// All arithmetic is float; only what the next product reads is in the storage type.
#include "common.h"
#include "api.h"
#include "recordable.h"

template <typename T> __device__ __forceinline__ void put4(T* p, f32x4 v);
template <> __device__ __forceinline__ void put4<float>(float* p, f32x4 v) { *(f32x4*)p = v; }
template <> __device__ __forceinline__ void put4<bf16_t>(bf16_t* p, f32x4 v) {
    bf16x4 o = {(bf16_t)v[0], (bf16_t)v[1], (bf16_t)v[2], (bf16_t)v[3]};
    *(bf16x4*)p = o;
}
template <typename T> __device__ __forceinline__ f32x4 get4(const T* p);
template <> __device__ __forceinline__ f32x4 get4<float>(const float* p) { return *(const f32x4*)p; }
template <> __device__ __forceinline__ f32x4 get4<bf16_t>(const bf16_t* p) {
    const bf16x4 v = *(const bf16x4*)p;
    return (f32x4){(float)v[0], (float)v[1], (float)v[2], (float)v[3]};
}

struct SublayerArgs {
    const float* y;              // [n][W], or with `place` the experts' rows [n * top][W]
    const int* place;            // [n * top] or null
    int top;
    const float* gate;           // [n][W] logits or null
    const float* gate_bias;      // [W] or null
    int centred;                 // the output's norm takes the mean off
    const float* w;              // [W]
    const float* b;              // [W] or null
    const float* scale;          // [W] or null
    float eps;
    float* resid;                // [n][W], read and written
    int next_centred;
    const float* next_w;         // [W] or null: no norm of the new stream
    const float* next_b;
    float next_eps;
    int W;
};

__device__ __forceinline__ float sublayer_gate(float z) { return 1.0f / (1.0f + expf(-z)); }

// A row's VPT groups of four values per thread stay in registers through both norms.  The number of threads follows
// from the row's length alone, so a row's bits do not depend on what else the step holds.
template <int NT, int VPT, typename TOut>
__global__ __launch_bounds__(NT) void sublayer_step_kernel(SublayerArgs a, TOut* __restrict__ out) {
    __shared__ float red[NT / 64];
    const int W = a.W;
    const size_t at = (size_t)blockIdx.x * W;
    f32x4 v[VPT], r[VPT];
    float s = 0.f;
#pragma unroll
    for (int k = 0; k < VPT; ++k) {
        const int i = 4 * (threadIdx.x + NT * k);
        v[k] = r[k] = (f32x4){0.f, 0.f, 0.f, 0.f};
        if (i >= W) continue;
        r[k] = *(const f32x4*)(a.resid + at + i);
        if (a.place) {
            for (int j = 0; j < a.top; ++j) v[k] += *(const f32x4*)(a.y + (size_t)a.place[(size_t)blockIdx.x * a.top + j] * W + i);
        } else {
            v[k] = *(const f32x4*)(a.y + at + i);
        }
        if (a.gate) {
            f32x4 z = *(const f32x4*)(a.gate + at + i);
            if (a.gate_bias) z += *(const f32x4*)(a.gate_bias + i);
#pragma unroll
            for (int e = 0; e < 4; ++e) v[k][e] *= sublayer_gate(z[e]);
        }
        s += (v[k][0] + v[k][1]) + (v[k][2] + v[k][3]);
    }
    auto statistics = [&](const f32x4* x, float sum, int centred, float eps, float& mean, float& inv) {
        mean = centred ? block_sum<NT / 64>(sum, red) / (float)W : 0.f;
        float q = 0.f;
#pragma unroll
        for (int k = 0; k < VPT; ++k)
            if (4 * (threadIdx.x + NT * k) < W) {
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const float d = x[k][e] - mean;
                    q = fmaf(d, d, q);
                }
            }
        inv = 1.0f / sqrtf(block_sum<NT / 64>(q, red) / (float)W + eps);
    };
    float mean, inv;
    statistics(v, s, a.centred, a.eps, mean, inv);
    s = 0.f;
#pragma unroll
    for (int k = 0; k < VPT; ++k) {
        const int i = 4 * (threadIdx.x + NT * k);
        if (i >= W) continue;
        const f32x4 w4 = *(const f32x4*)(a.w + i), b4 = a.b ? *(const f32x4*)(a.b + i) : (f32x4){0.f, 0.f, 0.f, 0.f};
        const f32x4 l4 = a.scale ? *(const f32x4*)(a.scale + i) : (f32x4){1.f, 1.f, 1.f, 1.f};
#pragma unroll
        for (int e = 0; e < 4; ++e) r[k][e] = fmaf(l4[e], fmaf((v[k][e] - mean) * inv, w4[e], b4[e]), r[k][e]);
        *(f32x4*)(a.resid + at + i) = r[k];
        s += (r[k][0] + r[k][1]) + (r[k][2] + r[k][3]);
    }
    if (!a.next_w) return;
    statistics(r, s, a.next_centred, a.next_eps, mean, inv);
#pragma unroll
    for (int k = 0; k < VPT; ++k) {
        const int i = 4 * (threadIdx.x + NT * k);
        if (i >= W) continue;
        const f32x4 w4 = *(const f32x4*)(a.next_w + i), b4 = a.next_b ? *(const f32x4*)(a.next_b + i) : (f32x4){0.f, 0.f, 0.f, 0.f};
        f32x4 o;
#pragma unroll
        for (int e = 0; e < 4; ++e) o[e] = fmaf((r[k][e] - mean) * inv, w4[e], b4[e]);
        put4<TOut>(out + at + i, o);
    }
}

// rows whose length is no multiple of four, or that are too long to be held
template <typename TOut>
__global__ __launch_bounds__(256) void sublayer_step_any_kernel(SublayerArgs a, TOut* __restrict__ out) {
    __shared__ float red[4];
    const int W = a.W;
    const size_t at = (size_t)blockIdx.x * W;
    auto value = [&](int i) {
        float v = 0.f;
        if (a.place) {
            for (int j = 0; j < a.top; ++j) v += a.y[(size_t)a.place[(size_t)blockIdx.x * a.top + j] * W + i];
        } else {
            v = a.y[at + i];
        }
        return a.gate ? v * sublayer_gate(a.gate[at + i] + (a.gate_bias ? a.gate_bias[i] : 0.f)) : v;
    };
    auto statistics = [&](auto&& x, int centred, float eps, float& mean, float& inv) {
        float s = 0.f, q = 0.f;
        mean = 0.f;
        if (centred) {
            for (int i = threadIdx.x; i < W; i += 256) s += x(i);
            mean = block_sum<4>(s, red) / (float)W;
        }
        for (int i = threadIdx.x; i < W; i += 256) {
            const float d = x(i) - mean;
            q = fmaf(d, d, q);
        }
        inv = 1.0f / sqrtf(block_sum<4>(q, red) / (float)W + eps);
    };
    float mean, inv;
    statistics(value, a.centred, a.eps, mean, inv);
    for (int i = threadIdx.x; i < W; i += 256)
        a.resid[at + i] = fmaf(a.scale ? a.scale[i] : 1.f, fmaf((value(i) - mean) * inv, a.w[i], a.b ? a.b[i] : 0.f), a.resid[at + i]);
    if (!a.next_w) return;
    statistics([&](int i) { return a.resid[at + i]; }, a.next_centred, a.next_eps, mean, inv);      // (a thread's own values)
    for (int i = threadIdx.x; i < W; i += 256)
        out[at + i] = from_f32<TOut>(fmaf((a.resid[at + i] - mean) * inv, a.next_w[i], a.next_b ? a.next_b[i] : 0.f));
}

extern "C" int fl_sublayer_step(const float* y, const int* place, int top, const float* gate, const float* gate_bias,
                                int centred, const float* w, const float* b, const float* scale, float eps, float* resid,
                                int next_centred, const float* next_w, const float* next_b, float next_eps, void* out,
                                int out_dtype, int n, int W, hipStream_t stream) {
    FL_CHECK(n >= 0 && W > 0 && y && w && resid && top >= 0, "sublayer_step: bad sizes or a missing tensor");
    FL_CHECK(!next_w || out, "sublayer_step: no place for the normed stream");
    FL_CHECK(!gate_bias || gate, "sublayer_step: a gate's bias without its logits");
    if (n == 0) return 0;
    const SublayerArgs a = {y, place, top, gate, gate_bias, centred, w, b, scale, eps, resid, next_centred, next_w, next_b, next_eps, W};
    auto aligned = [](const void* p) { return (uintptr_t)p % 16 == 0; };
    const bool whole = (W & 3) == 0 && W <= 4 * 1024 * 4 && aligned(y) && aligned(gate) && aligned(gate_bias) && aligned(w) && aligned(b) &&
                       aligned(scale) && aligned(resid) && aligned(next_w) && aligned(next_b) && aligned(out);
    auto run = [&](auto* o) {
        typedef typename std::remove_pointer<decltype(o)>::type T;
        if (!whole) sublayer_step_any_kernel<T><<<n, 256, 0, stream>>>(a, o);
        else if (W <= 4 * 64) sublayer_step_kernel<64, 1, T><<<n, 64, 0, stream>>>(a, o);
        else if (W <= 4 * 256) sublayer_step_kernel<256, 1, T><<<n, 256, 0, stream>>>(a, o);
        else if (W <= 4 * 512) sublayer_step_kernel<512, 1, T><<<n, 512, 0, stream>>>(a, o);
        else if (W <= 4 * 1024) sublayer_step_kernel<1024, 1, T><<<n, 1024, 0, stream>>>(a, o);
        else if (W <= 8 * 1024) sublayer_step_kernel<1024, 2, T><<<n, 1024, 0, stream>>>(a, o);
        else sublayer_step_kernel<1024, 4, T><<<n, 1024, 0, stream>>>(a, o);
    };
    if (!next_w || out_dtype == FL_F32) run((float*)out);
    else if (out_dtype == FL_BF16) run((bf16_t*)out);
    else FL_CHECK(false, "sublayer_step: unknown dtype %d", out_dtype);
    FL_LAUNCH_CHECK();
    return 0;
}
FL_RECORDABLE(fl_sublayer_step)

// ------------------------------------------------------------------ the convolution in front of a mixer
// h [n][C]; w [taps][C], the last tap the token's own; ring [slots][taps][C] float: the input of position p lies at
// p % taps, so that a step of one token writes a place it does not read, and running it twice changes nothing.  A
// request's first tokens of a step (those that reach behind it) and the ring itself belong to the threads of its first
// token, which read the ring before they write it; all other tokens read rows of the step only.
template <typename T, int VEC, int TAPS>          // TAPS 0: as many as `n_taps` says, in a loop that is not unrolled
__global__ __launch_bounds__(256) void input_conv_kernel(const T* __restrict__ h, const float* __restrict__ w, float* __restrict__ ring,
                                                         const int* __restrict__ positions, const int* __restrict__ tok_seq,
                                                         const int* __restrict__ seq_q_start, const int* __restrict__ seq_q_len,
                                                         const int* __restrict__ seq_slots, T* __restrict__ out, int C, int n_taps) {
    const int taps = TAPS > 0 ? TAPS : n_taps;
    const int c = (blockIdx.x * 256 + threadIdx.x) * VEC;
    if (c >= C) return;
    auto load = [&](const auto* p, float* v) {
        if constexpr (VEC == 4) {
            const f32x4 q = get4(p);
            v[0] = q[0]; v[1] = q[1]; v[2] = q[2]; v[3] = q[3];
        } else {
            v[0] = to_f32(*p);
        }
    };
    auto store = [&](auto* p, const float* v) {
        typedef typename std::remove_pointer<decltype(p)>::type TS;
        if constexpr (VEC == 4) put4<TS>(p, (f32x4){v[0], v[1], v[2], v[3]});
        else *p = from_f32<TS>(v[0]);
    };
    // one token's output; row(k) loads the input of tap k into its argument, or says that there is none
    auto token = [&](int t, auto&& row) {
        float acc[VEC], x[VEC], wk[VEC], own[VEC];
#pragma unroll
        for (int e = 0; e < VEC; ++e) acc[e] = 0.f;
#pragma unroll
        for (int k = 0; k < taps; ++k) {
            if (!row(k, x)) continue;
            load(w + (size_t)k * C + c, wk);
#pragma unroll
            for (int e = 0; e < VEC; ++e) acc[e] = fmaf(wk[e], x[e], acc[e]);
        }
        load(h + (size_t)t * C + c, own);
#pragma unroll
        for (int e = 0; e < VEC; ++e) acc[e] += own[e];
        store(out + (size_t)t * C + c, acc);
    };
    const int t = blockIdx.y, s = tok_seq[t], i = t - seq_q_start[s];
    if (i >= taps - 1 && i > 0) {
        token(t, [&](int k, float* x) { load(h + (size_t)(t - taps + 1 + k) * C + c, x); return true; });
    } else if (i == 0) {
        const int len = seq_q_len[s], slot = seq_slots[s], p0 = positions[t];
        float* mine = slot >= 0 ? ring + (size_t)slot * taps * C : nullptr;          // (rows that pad a batch have no slot)
        const int own = max(1, min(taps - 1, len));
        for (int j = 0; j < own; ++j)
            token(t + j, [&](int k, float* x) {
                const int p = p0 + j - taps + 1 + k;
                if (p < 0) return false;
                if (p >= p0) { load(h + (size_t)(t + p - p0) * C + c, x); return true; }
                if (!mine) return false;
                load(mine + (size_t)(p % taps) * C + c, x);
                return true;
            });
        if (mine && taps > 1)
            for (int j = max(0, len - taps + 1); j < len; ++j) {
                float x[VEC];
                load(h + (size_t)(t + j) * C + c, x);
                store(mine + (size_t)((p0 + j) % taps) * C + c, x);
            }
    }
}

extern "C" int fl_input_conv(const void* h, int dtype, const float* w, float* ring, const int* positions, const int* tok_seq,
                             const int* seq_q_start, const int* seq_q_len, const int* seq_slots, void* out, int n, int C,
                             int taps, hipStream_t stream) {
    FL_CHECK(n >= 0 && C > 0 && taps > 0 && h && w && out && h != out, "input_conv: bad sizes or a missing tensor");
    FL_CHECK(ring && positions && tok_seq && seq_q_start && seq_q_len && seq_slots, "input_conv: the requests' kept inputs are missing");
    if (n == 0) return 0;
    FL_CHECK(n <= 65535, "input_conv: %d rows are more than one grid takes", n);
    const bool vec = C % 4 == 0 && (uintptr_t)h % 16 == 0 && (uintptr_t)w % 16 == 0 && (uintptr_t)ring % 16 == 0 && (uintptr_t)out % 16 == 0;
    dim3 grid(ceil_div(C, 256 * (vec ? 4 : 1)), n);
#define FL_IC(T, V, N) input_conv_kernel<T, V, N><<<grid, 256, 0, stream>>>((const T*)h, w, ring, positions, tok_seq, seq_q_start, seq_q_len, seq_slots, (T*)out, C, taps)
#define FL_IC_N(T)                                                         \
    do {                                                                    \
        if (!vec) FL_IC(T, 1, 0);                                          \
        else if (taps == 2) FL_IC(T, 4, 2);                                \
        else if (taps == 3) FL_IC(T, 4, 3);                                \
        else if (taps == 4) FL_IC(T, 4, 4);                                \
        else FL_IC(T, 4, 0);                                               \
    } while (0)
    if (dtype == FL_F32) FL_IC_N(float);
    else if (dtype == FL_BF16) FL_IC_N(bf16_t);
    else FL_CHECK(false, "input_conv: unknown dtype %d", dtype);
#undef FL_IC_N
#undef FL_IC
    FL_LAUNCH_CHECK();
    return 0;
}
FL_RECORDABLE(fl_input_conv)

// ------------------------------------------------------------------ embedding with a row per pair of tokens
// out[t] = table[token] + pairs[row], row = (previous token * mul_prev + token * mul_cur) mod buckets, or `buckets` (the
// extra row behind them) at position 0.  last [slots][2]: the token of position p lies at p % 2, so that a step of one
// token writes the place it does not read.  A request's entry belongs to the block of its first token of the step,
// which reads it before it writes.
template <typename T>
__global__ __launch_bounds__(256) void embed_bigram_kernel(const T* __restrict__ table, const T* __restrict__ pairs,
                                                           const int* __restrict__ tokens, const int* __restrict__ positions,
                                                           const int* __restrict__ tok_seq, const int* __restrict__ seq_q_start,
                                                           const int* __restrict__ seq_q_len, const int* __restrict__ seq_slots,
                                                           int* __restrict__ last, float* __restrict__ out, int H, int V, int buckets,
                                                           long mul_prev, long mul_cur) {
    __shared__ int shared_prev;
    const int t = blockIdx.x, s = tok_seq[t], q0 = seq_q_start[s], pos = positions[t], slot = seq_slots[s];
    int tok = tokens[t];
    if (tok < 0 || tok >= V) tok = 0;           // the host rejects such ids before the launch
    if (threadIdx.x == 0) {
        int prev = t > q0 ? tokens[t - 1] : (slot >= 0 && pos > 0) ? last[2 * slot + ((pos - 1) & 1)] : 0;
        shared_prev = prev < 0 || prev >= V ? 0 : prev;
        if (t == q0 && slot >= 0) {
            const int len = seq_q_len[s];
            last[2 * slot + ((pos + len - 1) & 1)] = tokens[q0 + len - 1];
        }
    }
    __syncthreads();
    long row = buckets;
    if (pos > 0) {
        row = ((long)shared_prev * mul_prev + (long)tok * mul_cur) % buckets;
        if (row < 0) row += buckets;
    }
    for (int i = threadIdx.x; i < H; i += 256)
        out[(size_t)t * H + i] = to_f32(table[(size_t)tok * H + i]) + to_f32(pairs[(size_t)row * H + i]);
}

extern "C" int fl_embed_bigram(const void* table, const void* pairs, int dtype, const int* tokens, const int* positions,
                               const int* tok_seq, const int* seq_q_start, const int* seq_q_len, const int* seq_slots, int* last,
                               float* out, int n, int H, int V, int buckets, long mul_prev, long mul_cur, hipStream_t stream) {
    FL_CHECK(n >= 0 && H > 0 && V > 0 && buckets > 0 && last, "embed_bigram: bad sizes, or no place for the requests' last tokens");
    if (n == 0) return 0;
    if (dtype == FL_F32)
        embed_bigram_kernel<float><<<n, 256, 0, stream>>>((const float*)table, (const float*)pairs, tokens, positions, tok_seq, seq_q_start, seq_q_len, seq_slots, last, out, H, V, buckets, mul_prev, mul_cur);
    else if (dtype == FL_BF16)
        embed_bigram_kernel<bf16_t><<<n, 256, 0, stream>>>((const bf16_t*)table, (const bf16_t*)pairs, tokens, positions, tok_seq, seq_q_start, seq_q_len, seq_slots, last, out, H, V, buckets, mul_prev, mul_cur);
    else FL_CHECK(false, "embed_bigram: unknown dtype %d", dtype);
    FL_LAUNCH_CHECK();
    return 0;
}
FL_RECORDABLE(fl_embed_bigram)
