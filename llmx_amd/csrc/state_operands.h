// What a matrix-state recurrence makes of its projected rows as it reads them: silu of q, k and v, or a rotation of q and k
// (their first `dims` channels turn as pairs (i, i + dims/2) by the row's position).  All float32; every kernel of the
// recurrence goes through these functions, so a value is the same bits wherever it is read.
#pragma once
#include "common.h"

enum : int { STATE_OPERANDS_PLAIN = 0, STATE_OPERANDS_SILU = 1, STATE_OPERANDS_ROTATED = 2 };

struct StateOperands {
    const float* cos_sin;   // [positions, dims]: cos of the dims/2 pairs, then sin (ROTATED)
    const int* pos;         // [T]
    int dims;
};

__device__ __forceinline__ float silu_state(float v) { return v * (1.0f / (1.0f + expf(-v))); }

// Channel d of a q or k head whose values start at `head`, of the step's row `row`.
template <int KIND>
__device__ __forceinline__ float state_key(const StateOperands& o, const float* __restrict__ head, size_t row, int d) {
    const float x = head[d];
    if (KIND == STATE_OPERANDS_SILU) return silu_state(x);
    if (KIND == STATE_OPERANDS_ROTATED) {
        const int half = o.dims / 2;
        const bool turns = d < o.dims, first = d < half;
        const int i = turns ? (first ? d : d - half) : 0;
        const float y = head[turns ? (first ? d + half : i) : d];
        if (!turns) return x;
        const float* cs = o.cos_sin + (size_t)o.pos[row] * o.dims;
        const float c = cs[i], s = cs[half + i];
        return first ? fmaf(-y, s, x * c) : fmaf(y, s, x * c);
    }
    return x;
}
template <int KIND>
__device__ __forceinline__ float state_value(float v) { return KIND == STATE_OPERANDS_SILU ? silu_state(v) : v; }
