// What stands around the walk of a state-space mixer (the walk itself: fl_linear_scan_written).
//
//   fl_conv_steps        ahead of it: a causal convolution over time per channel with a bias and silu behind it, and the
//                        decay and the step of every (token, head): dt = softplus(z + dt_bias), decay = exp(-exp(A_log) dt)
//   fl_gated_group_norm  behind it: y silu(gate), then divided by its root mean square in equal parts, times a gain
//
// All arithmetic is float; only what the next product reads is in the storage type.
#include "common.h"
#include "api.h"
#include "recordable.h"

// ------------------------------------------------------------------ short convolution, steps and decays
struct ConvSteps {
    const float* proj; int ld, col0;      // the channels' inputs are the columns col0 .. col0 + C - 1
    const float* w;                       // [taps][C], the last tap the token's own
    const float* bias;                    // [C] or null
    float* ring; size_t slot_stride;      // per slot [taps][C]: the input of position p lies at p % taps
    const int* positions; const int* tok_seq; const int* seq_q_start; const int* seq_q_len; const int* seq_slots;
    float* out;                           // [n][C]
    int C, n_taps;
    int col_dt, H;                        // the steps' logits are the columns col_dt .. col_dt + H - 1
    const float* dt_bias; const float* a_log;
    float* gates;                         // [n][2 H]: decay, step
};

// A request's first tokens of a step (those that reach behind it) and its ring belong to the threads of its first
// token, which read the ring before they write it; all other tokens read rows of the step only.
template <int VEC, int TAPS>              // TAPS 0: as many as n_taps says, in a loop that is not unrolled
__global__ __launch_bounds__(256) void conv_steps_kernel(ConvSteps a) {
    const int taps = TAPS > 0 ? TAPS : a.n_taps;
    const int t = blockIdx.y;
    if (blockIdx.x == 0)
        for (int h = threadIdx.x; h < a.H; h += 256) {
            const float z = a.proj[(size_t)t * a.ld + a.col_dt + h] + a.dt_bias[h];
            const float dt = fmaxf(z, 0.f) + log1pf(expf(-fabsf(z)));
            a.gates[(size_t)t * 2 * a.H + h] = expf(-expf(a.a_log[h]) * dt);
            a.gates[(size_t)t * 2 * a.H + a.H + h] = dt;
        }
    const int C = a.C, c = (blockIdx.x * 256 + threadIdx.x) * VEC;
    if (c >= C) return;
    auto load = [&](const float* p, float* v) {
        if constexpr (VEC == 4) {
            const f32x4 q = *(const f32x4*)p;
            v[0] = q[0]; v[1] = q[1]; v[2] = q[2]; v[3] = q[3];
        } else {
            v[0] = *p;
        }
    };
    auto store = [&](float* p, const float* v) {
        if constexpr (VEC == 4) *(f32x4*)p = (f32x4){v[0], v[1], v[2], v[3]};
        else *p = v[0];
    };
    auto input = [&](int row) { return a.proj + (size_t)row * a.ld + a.col0 + c; };
    // one token's output; row(k) loads the input of tap k into its argument, or says that there is none
    auto token = [&](int row_out, auto&& row) {
        float acc[VEC], x[VEC], wk[VEC];
#pragma unroll
        for (int e = 0; e < VEC; ++e) acc[e] = 0.f;
        if (a.bias) load(a.bias + c, acc);
#pragma unroll
        for (int k = 0; k < taps; ++k) {
            if (!row(k, x)) continue;
            load(a.w + (size_t)k * C + c, wk);
#pragma unroll
            for (int e = 0; e < VEC; ++e) acc[e] = fmaf(wk[e], x[e], acc[e]);
        }
#pragma unroll
        for (int e = 0; e < VEC; ++e) acc[e] = acc[e] / (1.0f + expf(-acc[e]));
        store(a.out + (size_t)row_out * C + c, acc);
    };
    const int s = a.tok_seq[t], i = t - a.seq_q_start[s];
    if (i >= taps - 1 && i > 0) {
        token(t, [&](int k, float* x) { load(input(t - taps + 1 + k), x); return true; });
    } else if (i == 0) {
        const int len = a.seq_q_len[s], slot = a.seq_slots[s], p0 = a.positions[t];
        float* mine = slot >= 0 ? a.ring + (size_t)slot * a.slot_stride : nullptr;       // (rows that pad a batch have no slot)
        const int own = max(1, min(taps - 1, len));
        for (int j = 0; j < own; ++j)
            token(t + j, [&](int k, float* x) {
                const int p = p0 + j - taps + 1 + k;
                if (p < 0) return false;
                if (p >= p0) { load(input(t + p - p0), x); return true; }
                if (!mine) return false;
                load(mine + (size_t)(p % taps) * C + c, x);
                return true;
            });
        if (mine && taps > 1)
            for (int j = max(0, len - taps + 1); j < len; ++j) {
                float x[VEC];
                load(input(t + j), x);
                store(mine + (size_t)((p0 + j) % taps) * C + c, x);
            }
    }
}

extern "C" int fl_conv_steps(const float* proj, int ld, int col0, const float* w, const float* bias, float* ring, long slot_stride,
                             const int* positions, const int* tok_seq, const int* seq_q_start, const int* seq_q_len,
                             const int* seq_slots, float* out, int n, int C, int taps, int col_dt, int H, const float* dt_bias,
                             const float* a_log, float* gates, hipStream_t stream) {
    FL_CHECK(n >= 0 && C > 0 && taps > 0 && H > 0 && col0 >= 0 && col_dt >= 0, "conv_steps: bad sizes");
    FL_CHECK(ld >= col0 + C && ld >= col_dt + H, "conv_steps: columns beyond rows %d wide", ld);
    FL_CHECK(proj && w && ring && out && dt_bias && a_log && gates, "conv_steps: a missing tensor");
    FL_CHECK(slot_stride >= (long)taps * C, "conv_steps: a slot of %ld floats does not hold %d inputs of %d channels", slot_stride, taps, C);
    if (n == 0) return 0;
    FL_CHECK(n <= 65535, "conv_steps: %d rows are more than one grid takes", n);
    const ConvSteps a{proj, ld, col0, w, bias, ring, (size_t)slot_stride, positions, tok_seq, seq_q_start, seq_q_len, seq_slots, out,
                      C, taps, col_dt, H, dt_bias, a_log, gates};
    auto aligned = [](const void* p) { return (uintptr_t)p % 16 == 0; };
    const bool vec = C % 4 == 0 && ld % 4 == 0 && col0 % 4 == 0 && slot_stride % 4 == 0 && aligned(proj) && aligned(w) && aligned(bias) &&
                     aligned(ring) && aligned(out);
    dim3 grid(ceil_div(C, 256 * (vec ? 4 : 1)), n);
    if (!vec) conv_steps_kernel<1, 0><<<grid, 256, 0, stream>>>(a);
    else if (taps == 2) conv_steps_kernel<4, 2><<<grid, 256, 0, stream>>>(a);
    else if (taps == 3) conv_steps_kernel<4, 3><<<grid, 256, 0, stream>>>(a);
    else if (taps == 4) conv_steps_kernel<4, 4><<<grid, 256, 0, stream>>>(a);
    else conv_steps_kernel<4, 0><<<grid, 256, 0, stream>>>(a);
    FL_LAUNCH_CHECK();
    return 0;
}
FL_RECORDABLE(fl_conv_steps)

// ------------------------------------------------------------------ a gate, then a norm in equal parts
// out[t][p * P + i] = v / sqrt(mean over the part of v^2 + eps) * w[p * P + i], v = y silu(gate): a block per (token, part of P
// values).  A part of up to 256 * HELD values is formed once and stays in registers.
template <typename T, int HELD>
__global__ __launch_bounds__(256) void gated_group_norm_kernel(const float* __restrict__ y, const float* __restrict__ gate, int ldg,
                                                               int gate_col0, const float* __restrict__ w, T* __restrict__ out,
                                                               int ldo, int W, int P, float eps) {
    __shared__ float lds[4];
    const size_t t = blockIdx.x;
    const int at = blockIdx.y * P;
    const float* yr = y + t * W + at;
    const float* zr = gate + t * ldg + gate_col0 + at;
    auto value = [&](int i) {
        const float z = zr[i];
        return yr[i] * (z / (1.0f + expf(-z)));
    };
    float v[HELD > 0 ? HELD : 1], ss = 0.f;
    if constexpr (HELD > 0) {
#pragma unroll
        for (int k = 0; k < HELD; ++k) {
            const int i = threadIdx.x + 256 * k;
            v[k] = i < P ? value(i) : 0.f;
            ss = fmaf(v[k], v[k], ss);
        }
    } else {
        for (int i = threadIdx.x; i < P; i += 256) {
            const float u = value(i);
            ss = fmaf(u, u, ss);
        }
    }
    const float inv = 1.0f / sqrtf(block_sum<4>(ss, lds) / (float)P + eps);
    T* dst = out + t * ldo + at;
    if constexpr (HELD > 0) {
#pragma unroll
        for (int k = 0; k < HELD; ++k) {
            const int i = threadIdx.x + 256 * k;
            if (i < P) dst[i] = from_f32<T>(v[k] * inv * w[at + i]);
        }
    } else {
        for (int i = threadIdx.x; i < P; i += 256) dst[i] = from_f32<T>(value(i) * inv * w[at + i]);
    }
}

extern "C" int fl_gated_group_norm(const float* y, const float* gate, int ldg, int gate_col0, const float* w, void* out,
                                   int out_dtype, int ldo, int n, int W, int parts, float eps, hipStream_t stream) {
    FL_CHECK(n >= 0 && W > 0 && parts > 0 && W % parts == 0 && gate_col0 >= 0 && y && gate && w && out, "gated_group_norm: %d values in %d parts, or a missing tensor", W, parts);
    FL_CHECK(ldg >= gate_col0 + W && ldo >= W, "gated_group_norm: gate rows of %d, output rows of %d values", ldg, ldo);
    if (n == 0) return 0;
    FL_CHECK(parts <= 65535, "gated_group_norm: %d parts are more than one grid takes", parts);
    const int P = W / parts;
    dim3 grid(n, parts);
#define FL_GGN(T, K) gated_group_norm_kernel<T, K><<<grid, 256, 0, stream>>>(y, gate, ldg, gate_col0, w, (T*)out, ldo, W, P, eps)
#define FL_GGN_K(T)                       \
    do {                                  \
        if (P <= 256) FL_GGN(T, 1);       \
        else if (P <= 1024) FL_GGN(T, 4); \
        else if (P <= 4096) FL_GGN(T, 16);\
        else FL_GGN(T, 0);                \
    } while (0)
    if (out_dtype == FL_F32) FL_GGN_K(float);
    else if (out_dtype == FL_BF16) FL_GGN_K(bf16_t);
    else FL_CHECK(false, "gated_group_norm: unknown dtype %d", out_dtype);
#undef FL_GGN_K
#undef FL_GGN
    FL_LAUNCH_CHECK();
    return 0;
}
FL_RECORDABLE(fl_gated_group_norm)
