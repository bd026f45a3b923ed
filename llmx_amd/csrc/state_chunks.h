// The parts that the chunk-by-chunk forms of the matrix-state recurrences share: a chunk's rows of one head on their way into LDS,
// and the read-out of a chunk's rows from the state before it and the chunk's own outer products,
//     o_i = upto(i) S^T q_i + sum_(j <= i) between(i, j) (q_i . k_j) v_j
// with the decays upto (the state's, at row i) and between (row j's product's, at row i) of the recurrence.
// 16x16x4 instructions (A: row lane % 16, k lane / 16; B: column lane % 16, k lane / 16; the result: rows 4 (lane / 16) + 0..3 of
// column lane % 16).  The 4 k-slots of an instruction are dealt so that a lane's operands of four instructions are 16
// neighbouring bytes.
#pragma once
#include "state_operands.h"

typedef float f32x4_t __attribute__((ext_vector_type(4)));

#define DS_ROWS 64       // rows of a chunk

// One head's rows of one chunk: row j of the chunk at q + j ldq, k + j ldk, v + j ldv, out + j ldo.
struct ChunkRows {
    const float* q;
    const float* k;
    const float* v;
    int ldq, ldk, ldv;
    int row0, n;               // the chunk's first row in the step (for its position), its rows
    int D, V, DR, VR;          // channels, and the same in whole tiles of 16
    const float* start;        // [VR][DR]: the state before the chunk
    float* out;
    int ldo;
    float out_scale;
    StateOperands operands;
};

__device__ __forceinline__ f32x4_t mfma4(float a, float b, f32x4_t c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

// A chunk's keys into LDS rows of LDK floats (channels from D on and rows from n on hold zeros).  VEC: 16-byte loads, as many in
// flight as a thread has to bring (see state_keys4_load for what they ask for); otherwise value by value.
template <int NU, int KIND, bool VEC, int LDK>
__device__ __forceinline__ void stage_keys(const ChunkRows& a, float* ks) {
    constexpr int DP = 16 * NU;
    const int tid = threadIdx.x;
    if (VEC) {
        constexpr int PER_ROW = DP / 4, PER_THREAD = DS_ROWS * PER_ROW / 256, TURN = PER_THREAD < 8 ? PER_THREAD : 8;
#pragma unroll
        for (int b = 0; b < PER_THREAD; b += TURN) {
            StateKeys4 raw[TURN];
#pragma unroll
            for (int u = 0; u < TURN; ++u) {
                const int i = tid + 256 * (b + u), j = i / PER_ROW, d = 4 * (i % PER_ROW);
                const size_t row = (size_t)min(j, a.n - 1);
                raw[u] = state_keys4_load<KIND>(a.operands, a.k + row * a.ldk, a.row0 + row, d < a.D ? d : 0);
            }
#pragma unroll
            for (int u = 0; u < TURN; ++u) {
                const int i = tid + 256 * (b + u), j = i / PER_ROW, d = 4 * (i % PER_ROW);
                const state4_t x = state_keys4<KIND>(raw[u]);
                *reinterpret_cast<state4_t*>(ks + j * LDK + d) = d < a.D && j < a.n ? x : state4_t{0.0f, 0.0f, 0.0f, 0.0f};
            }
        }
        return;
    }
    for (int i = tid; i < DS_ROWS * DP; i += 256) {
        const int j = i / DP, d = i % DP;
        const size_t row = (size_t)min(j, a.n - 1);
        const float x = state_key<KIND>(a.operands, a.k + row * a.ldk, a.row0 + row, min(d, a.D - 1));
        ks[j * LDK + d] = d < a.D && j < a.n ? x : 0.0f;
    }
}

// 64 value channels from v0 on of a chunk's rows, row j times weight(j).
template <int KIND, bool VEC, int LDV, typename Weight>
__device__ __forceinline__ void stage_values(const ChunkRows& a, int v0, float* vs, Weight weight) {
    const int tid = threadIdx.x;
    if (VEC) {
        state4_t raw[4];
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            const int i = tid + 256 * u, j = i / 16, v = v0 + 4 * (i % 16);
            raw[u] = *reinterpret_cast<const state4_t*>(a.v + (size_t)min(j, a.n - 1) * a.ldv + (v < a.V ? v : 0));
        }
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            const int i = tid + 256 * u, j = i / 16, v = v0 + 4 * (i % 16);
            const float w = j < a.n ? weight(j) : 0.0f;
            state4_t x;
#pragma unroll
            for (int e = 0; e < 4; ++e) x[e] = v < a.V && j < a.n ? state_value<KIND>(raw[u][e]) * w : 0.0f;
            *reinterpret_cast<state4_t*>(vs + j * LDV + 4 * (i % 16)) = x;
        }
        return;
    }
    for (int i = tid; i < DS_ROWS * 64; i += 256) {
        const int j = i / 64, v = v0 + i % 64;
        const float x = state_value<KIND>(a.v[(size_t)min(j, a.n - 1) * a.ldv + min(v, a.V - 1)]);
        vs[j * LDV + i % 64] = v < a.V && j < a.n ? x * weight(j) : 0.0f;
    }
}

// The read-out of a chunk's rows by a workgroup of four waves.  `decay` is ready for use by every thread once the first barrier
// in here has passed.  Floats of LDS: state_rows_lds(NU).
constexpr size_t state_rows_lds(int NU) { return DS_ROWS * (size_t)(16 * NU + 4 + 64 + 4); }
template <int NU, int KIND, bool VEC, typename Decay>
__device__ __forceinline__ void state_rows_read(const ChunkRows& a, const Decay& decay, float* lds) {
    constexpr int DP = 16 * NU, LDK = DP + 4, LDV = 64 + 4;
    float* ks = lds;                       // [64][LDK]: keys, then the state's value channels (64 at a time)
    float* vs = lds + DS_ROWS * LDK;       // [64][LDV]
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, c = lane & 15, g = lane >> 4;
    const int n = a.n;

    // the wave's 16 query rows, in registers: lane (c, g) holds row 16 wave + c, channels 16 u + 4 g + 0..3
    f32x4_t q[NU];
    {
        const size_t row = (size_t)(a.row0 + min(16 * wave + c, n - 1));
        const float* head = a.q + (size_t)min(16 * wave + c, n - 1) * a.ldq;
        if (VEC) {
            constexpr int TURN = NU < 8 ? NU : 8;
#pragma unroll
            for (int b = 0; b < NU; b += TURN) {
                StateKeys4 raw[TURN];
#pragma unroll
                for (int u = 0; u < TURN; ++u) {
                    const int d = 16 * (b + u) + 4 * g;
                    raw[u] = state_keys4_load<KIND>(a.operands, head, row, d < a.D ? d : 0);
                }
#pragma unroll
                for (int u = 0; u < TURN; ++u) {
                    const state4_t x = state_keys4<KIND>(raw[u]);
                    q[b + u] = 16 * (b + u) + 4 * g < a.D ? x : state4_t{0.0f, 0.0f, 0.0f, 0.0f};
                }
            }
        } else {
#pragma unroll
            for (int u = 0; u < NU; ++u)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const int d = 16 * u + 4 * g + e;
                    const float x = state_key<KIND>(a.operands, head, row, min(d, a.D - 1));
                    q[u][e] = d < a.D ? x : 0.0f;
                }
        }
    }
    stage_keys<NU, KIND, VEC, LDK>(a, ks);
    __syncthreads();
    // scores transposed: s[t][e] of key row 16 t + 4 g + e against query row 16 wave + c, t up to the wave's own tile
    f32x4_t s[4];
#pragma unroll
    for (int t = 0; t < 4; ++t) s[t] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
    for (int u = 0; u < NU; ++u) {
#pragma unroll
        for (int t = 0; t < 4; ++t) {
            if (t <= wave) {
                const f32x4_t kf = *reinterpret_cast<const f32x4_t*>(ks + (16 * t + c) * LDK + 16 * u + 4 * g);
#pragma unroll
                for (int e = 0; e < 4; ++e) s[t] = mfma4(kf[e], q[u][e], s[t]);
            }
        }
    }
    const int i_row = 16 * wave + c;
#pragma unroll
    for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int j_row = 16 * t + 4 * g + e;
            s[t][e] = j_row <= i_row ? s[t][e] * decay.between(i_row, j_row) : 0.0f;
        }
    const float* start = a.start;
    for (int v0 = 0; v0 < a.VR; v0 += 64) {
        __syncthreads();       // the keys, or the slice before, have been read by every wave
        {
            constexpr int PER_ROW = DP / 4, PER_THREAD = 64 * PER_ROW / 256, TURN = PER_THREAD < 8 ? PER_THREAD : 8;
#pragma unroll
            for (int b = 0; b < PER_THREAD; b += TURN) {
                f32x4_t x[TURN];
#pragma unroll
                for (int u = 0; u < TURN; ++u) {
                    const int i = tid + 256 * (b + u), v = i / PER_ROW, d = 4 * (i % PER_ROW);
                    const bool in = v0 + v < a.VR && d < a.DR;
                    x[u] = *reinterpret_cast<const f32x4_t*>(start + (size_t)(in ? v0 + v : 0) * a.DR + (in ? d : 0));
                    if (!in) x[u] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
                }
#pragma unroll
                for (int u = 0; u < TURN; ++u) {
                    const int i = tid + 256 * (b + u);
                    *reinterpret_cast<f32x4_t*>(ks + (i / PER_ROW) * LDK + 4 * (i % PER_ROW)) = x[u];
                }
            }
        }
        stage_values<KIND, VEC, LDV>(a, v0, vs, [](int) { return 1.0f; });
        __syncthreads();
        f32x4_t o[4];
#pragma unroll
        for (int t = 0; t < 4; ++t) o[t] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
        for (int u = 0; u < NU; ++u)
#pragma unroll
            for (int vt = 0; vt < 4; ++vt) {
                const f32x4_t sf = *reinterpret_cast<const f32x4_t*>(ks + (16 * vt + c) * LDK + 16 * u + 4 * g);
#pragma unroll
                for (int e = 0; e < 4; ++e) o[vt] = mfma4(q[u][e], sf[e], o[vt]);
            }
        // o[vt][e]: row 16 wave + 4 g + e, value channel v0 + 16 vt + c
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const float keep = decay.upto(16 * wave + 4 * g + e);
#pragma unroll
            for (int vt = 0; vt < 4; ++vt) o[vt][e] *= keep;
        }
#pragma unroll
        for (int t = 0; t < 4; ++t) {
            if (t <= wave) {
#pragma unroll
                for (int e = 0; e < 4; ++e)
#pragma unroll
                    for (int vt = 0; vt < 4; ++vt) o[vt] = mfma4(s[t][e], vs[(16 * t + 4 * g + e) * LDV + 16 * vt + c], o[vt]);
            }
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int i = 16 * wave + 4 * g + e;
            if (i < n) {
                float* to = a.out + (size_t)i * a.ldo;
#pragma unroll
                for (int vt = 0; vt < 4; ++vt) {
                    const int v = v0 + 16 * vt + c;
                    if (v < a.V) to[v] = o[vt][e] * a.out_scale;
                }
            }
        }
    }
}

