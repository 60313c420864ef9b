// The rotated part of a query or key that stands behind a latent (latent.hip, latent_tuned.hip).
#pragma once
#include "common.h"

// Dimension i of a part v whose first `rot` dims are turned by the token's angles, i with i + rot / 2 or (interleaved)
// 2i with 2i + 1: cs [rot / 2][2] cosines and sines.
__device__ __forceinline__ float rotated_value(const float* v, int i, int rot, int interleaved, const float* cs) {
    if (i >= rot) return v[i];
    const int half = rot >> 1;
    const int pair = interleaved ? i >> 1 : i < half ? i : i - half;
    const bool first = interleaved ? !(i & 1) : i < half;
    const float a = v[interleaved ? 2 * pair : pair], b = v[interleaved ? 2 * pair + 1 : pair + half];
    const float c = cs[2 * pair], s = cs[2 * pair + 1];
    return first ? a * c - b * s : b * c + a * s;
}

// What stands behind a head's folded query: `width` values, zeros but for the head's rotated part of rot_dim values,
// which begins at `at`; the part as the projection left it lies at column `col` of the head's row.
struct QueryTail {
    int width, col, at, rot_dim, rot, interleaved;
    const float* cs;                    // [tokens][rot / 2][2]
};

__device__ __forceinline__ float query_tail_value(const QueryTail& t, const float* head_row, int token, int d) {
    const int i = d - t.at;
    if (i < 0 || i >= t.rot_dim) return 0.f;
    return rotated_value(head_row + t.col, i, t.rot, t.interleaved, t.cs + (size_t)token * t.rot);
}
