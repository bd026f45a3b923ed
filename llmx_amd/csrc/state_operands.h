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
// Channels d .. d + 3 of such a head, d a multiple of 4 below D, with 16-byte loads: the head's start, its row stride and D are
// multiples of 4 floats, and so is dims / 2.  The same operations as state_key.
typedef float state4_t __attribute__((ext_vector_type(4)));
struct StateKeys4 {
    state4_t x, y, c, s;      // the channels, their partners, cos and sin of their pairs: asked for together, used later
    bool turns, first;
};
template <int KIND>
__device__ __forceinline__ StateKeys4 state_keys4_load(const StateOperands& o, const float* __restrict__ head, size_t row, int d) {
    StateKeys4 k;
    k.x = *reinterpret_cast<const state4_t*>(head + d);
    if (KIND == STATE_OPERANDS_ROTATED) {
        const int half = o.dims / 2;
        k.turns = d < o.dims;
        k.first = d < half;
        const int i = k.turns ? (k.first ? d : d - half) : 0;
        const float* cs = o.cos_sin + (size_t)o.pos[row] * o.dims;
        k.y = *reinterpret_cast<const state4_t*>(head + (k.turns ? (k.first ? d + half : i) : d));
        k.c = *reinterpret_cast<const state4_t*>(cs + i);
        k.s = *reinterpret_cast<const state4_t*>(cs + half + i);
    }
    return k;
}
template <int KIND>
__device__ __forceinline__ state4_t state_keys4(const StateKeys4& k) {
    state4_t r = k.x;
    if (KIND == STATE_OPERANDS_SILU) {
#pragma unroll
        for (int e = 0; e < 4; ++e) r[e] = silu_state(k.x[e]);
    }
    if (KIND == STATE_OPERANDS_ROTATED) {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const float turned = k.first ? fmaf(-k.y[e], k.s[e], k.x[e] * k.c[e]) : fmaf(k.y[e], k.s[e], k.x[e] * k.c[e]);
            r[e] = k.turns ? turned : k.x[e];
        }
    }
    return r;
}
template <int KIND>
__device__ __forceinline__ float state_value(float v) { return KIND == STATE_OPERANDS_SILU ? silu_state(v) : v; }
