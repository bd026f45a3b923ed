// The matrix-state recurrence with one constant decay g a head,
//     S_t = g S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t,
// for long runs of rows, chunk by chunk on the float32 matrix instruction (short runs: state_scan of linear_state.hip; the
// two differ by rounding).  With i, j counting a chunk's n rows from 0 and S the state before it,
//     o_i = g^(i+1) S^T q_i + sum_(j <= i) g^(i-j) (q_i . k_j) v_j,      S <- g^n S + sum_j g^(n-1-j) k_j v_j^T,
// every power of g at most 1, taken from a table that the host forms in float64.  Three launches:
//   sums    a workgroup a (chunk, head, 64 value channels): the chunk's own sum_j g^(n-1-j) k_j v_j^T into `starts`;
//   starts  a thread 4 key channels of a (head, value channel): walks the request's chunks in order from its state slot, leaves in
//           `starts` the state before each chunk and writes the last state to the request's slot;
//   rows    a workgroup a (chunk, head): scores, the decayed causal weights, the read-out of the state and the value product.
// Everything is float32.
// starts: [chunk][head][value channel, padded to 16][key channel, padded to 16].
#include "state_chunks.h"

struct DecayedArgs {
    const float* q;
    const float* k;
    const float* v;
    int ldq, ldk, ldv;
    const float* powers;       // [H, DS_ROWS + 1]: g^0 .. g^DS_ROWS
    float* state;              // S at the slot's start, in the scan's tiles: [H, ceil(V / 8), D, 8]
    long state_stride;
    const int* slot_read;
    const int* slot_write;
    const int* chunks;         // [n_chunks, 4]: entry, first row, rows, -
    const int* entry_chunks;   // [n_long, 4]: entry, first chunk, chunks, -
    float* starts;
    float* out;                // [T, H * V]
    float out_scale;
    int H, D, V, DR, VR;
    StateOperands operands;
};

// The rows of chunk blockIdx.x and head blockIdx.y.
__device__ __forceinline__ ChunkRows chunk_rows(const DecayedArgs& a) {
    const int* chunk = a.chunks + 4 * (size_t)blockIdx.x;
    const int row0 = chunk[1], n = chunk[2], h = blockIdx.y;
    return ChunkRows{a.q + (size_t)row0 * a.ldq + (size_t)h * a.D, a.k + (size_t)row0 * a.ldk + (size_t)h * a.D,
                     a.v + (size_t)row0 * a.ldv + (size_t)h * a.V, a.ldq, a.ldk, a.ldv, row0, n, a.D, a.V, a.DR, a.VR,
                     a.starts + ((size_t)blockIdx.x * a.H + h) * a.VR * a.DR, a.out + (size_t)row0 * a.H * a.V + (size_t)h * a.V, a.H * a.V,
                     a.out_scale, a.operands};
}

// NU: a head's key channels in tiles of 16, padded
template <int NU, int KIND, bool VEC>
__global__ void __launch_bounds__(256) decayed_sums_kernel(DecayedArgs a) {
    constexpr int DP = 16 * NU, LDK = DP + 16, LDV = 64 + 16;     // rows 16 banks apart: four rows' 16 neighbours meet no bank twice
    extern __shared__ __align__(16) float lds[];
    float* ks = lds;                       // [64][LDK]
    float* vs = lds + DS_ROWS * LDK;       // [64][LDV]: values times g^(n-1-j)
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, c = lane & 15, g = lane >> 4;
    const ChunkRows rows = chunk_rows(a);
    const int n = rows.n, h = blockIdx.y, v0 = 64 * blockIdx.z;
    const float* pw = a.powers + (size_t)h * (DS_ROWS + 1);
    const int steps = (n + 3) / 4;
    stage_values<KIND, VEC, LDV>(rows, v0, vs, [&](int j) { return pw[n - 1 - j]; });
    stage_keys<NU, KIND, VEC, LDK>(rows, ks);
    __syncthreads();
    if (v0 + 16 * wave >= a.VR) return;
    f32x4_t acc[NU];
#pragma unroll
    for (int u = 0; u < NU; ++u) acc[u] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
    for (int s = 0; s < steps; ++s) {
        const float b = vs[(4 * s + g) * LDV + 16 * wave + c];
#pragma unroll
        for (int u = 0; u < NU; ++u) acc[u] = mfma4(ks[(4 * s + g) * LDK + 16 * u + c], b, acc[u]);
    }
    // acc[u][e]: key channel 16 u + 4 g + e, value channel v0 + 16 wave + c
    float* to = a.starts + (((size_t)blockIdx.x * a.H + h) * a.VR + v0 + 16 * wave + c) * a.DR + 4 * g;
#pragma unroll
    for (int u = 0; u < NU; ++u)
        if (16 * u < a.DR) *reinterpret_cast<f32x4_t*>(to + 16 * u) = acc[u];
}

#define DS_AHEAD 8       // chunks whose sums are on their way together
__global__ void __launch_bounds__(256) decayed_starts_kernel(DecayedArgs a) {
    const int per_head = a.VR * a.DR / 4;
    const int at = blockIdx.x * 256 + threadIdx.x;
    if (at >= a.H * per_head) return;
    const int h = at / per_head, rem = at % per_head, v = rem / (a.DR / 4), d = 4 * (rem % (a.DR / 4));
    const int* ec = a.entry_chunks + 4 * (size_t)blockIdx.y;
    const int e = ec[0], c0 = ec[1], nc = ec[2];
    const int tiles = (a.V + 7) / 8;
    const size_t tile_at = ((size_t)h * tiles + v / 8) * a.D * 8 + (size_t)d * 8 + v % 8;
    const float* from = a.state + (size_t)a.slot_read[e] * a.state_stride + tile_at;
    float* to = a.state + (size_t)a.slot_write[e] * a.state_stride + tile_at;
    const float* pw = a.powers + (size_t)h * (DS_ROWS + 1);
    f32x4_t S;
#pragma unroll
    for (int i = 0; i < 4; ++i) S[i] = v < a.V && d + i < a.D ? from[8 * i] : 0.0f;
    const size_t stride = (size_t)a.H * a.VR * a.DR;
    float* p = a.starts + (size_t)c0 * stride + (size_t)h * a.VR * a.DR + (size_t)v * a.DR + d;
    for (int b = 0; b < nc; b += DS_AHEAD) {
        f32x4_t sum[DS_AHEAD];
        float keep[DS_AHEAD];
#pragma unroll
        for (int i = 0; i < DS_AHEAD; ++i) {
            const int k = min(b + i, nc - 1);
            sum[i] = *reinterpret_cast<const f32x4_t*>(p + (size_t)k * stride);
            keep[i] = pw[a.chunks[4 * (size_t)(c0 + k) + 2]];
        }
#pragma unroll
        for (int i = 0; i < DS_AHEAD; ++i) {
            if (b + i < nc) {
                *reinterpret_cast<f32x4_t*>(p + (size_t)(b + i) * stride) = S;
#pragma unroll
                for (int x = 0; x < 4; ++x) S[x] = fmaf(keep[i], S[x], sum[i][x]);
            }
        }
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
        if (v < a.V && d + i < a.D) to[8 * i] = S[i];
}

// The decays of one head from the table of its decay's powers.
struct PowerDecay {
    const float* pw;           // [65] in LDS: g^0 .. g^64
    __device__ __forceinline__ float between(int i, int j) const { return pw[i - j]; }
    __device__ __forceinline__ float upto(int i) const { return pw[i + 1]; }
};

template <int NU, int KIND, bool VEC>
__global__ void __launch_bounds__(256) decayed_rows_kernel(DecayedArgs a) {
    extern __shared__ __align__(16) float lds[];
    float* pw = lds + state_rows_lds(NU);
    const ChunkRows rows = chunk_rows(a);
    for (int i = threadIdx.x; i <= DS_ROWS; i += 256) pw[i] = a.powers[(size_t)blockIdx.y * (DS_ROWS + 1) + i];
    state_rows_read<NU, KIND, VEC>(rows, PowerDecay{pw}, lds);
}

template <int NU, int KIND, bool VEC>
static int launch_decayed(const DecayedArgs& a, int n_chunks, int n_long, hipStream_t stream) {
    constexpr size_t lds_sums = sizeof(float) * DS_ROWS * (16 * NU + 16 + 64 + 16);
    constexpr size_t lds_rows = sizeof(float) * (state_rows_lds(NU) + DS_ROWS + 1);
    static bool raised = false;
    if (!raised) {
        if (hipFuncSetAttribute((const void*)decayed_sums_kernel<NU, KIND, VEC>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024) != hipSuccess) return -1;
        if (hipFuncSetAttribute((const void*)decayed_rows_kernel<NU, KIND, VEC>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024) != hipSuccess) return -1;
        raised = true;
    }
    hipLaunchKernelGGL((decayed_sums_kernel<NU, KIND, VEC>), dim3(n_chunks, a.H, (a.VR + 63) / 64), dim3(256), lds_sums, stream, a);
    hipLaunchKernelGGL(decayed_starts_kernel, dim3((unsigned)(((size_t)a.H * a.VR * a.DR / 4 + 255) / 256), n_long), dim3(256), 0, stream, a);
    hipLaunchKernelGGL((decayed_rows_kernel<NU, KIND, VEC>), dim3(n_chunks, a.H), dim3(256), lds_rows, stream, a);
    return LLMX_CHECK_LAUNCH();
}

template <int NU>
static int launch_decayed_kind(const DecayedArgs& a, int kind, bool vec, int n_chunks, int n_long, hipStream_t stream) {
    if (kind == STATE_OPERANDS_SILU)
        return vec ? launch_decayed<NU, STATE_OPERANDS_SILU, true>(a, n_chunks, n_long, stream) : launch_decayed<NU, STATE_OPERANDS_SILU, false>(a, n_chunks, n_long, stream);
    if (kind == STATE_OPERANDS_ROTATED)
        return vec ? launch_decayed<NU, STATE_OPERANDS_ROTATED, true>(a, n_chunks, n_long, stream) : launch_decayed<NU, STATE_OPERANDS_ROTATED, false>(a, n_chunks, n_long, stream);
    return vec ? launch_decayed<NU, STATE_OPERANDS_PLAIN, true>(a, n_chunks, n_long, stream) : launch_decayed<NU, STATE_OPERANDS_PLAIN, false>(a, n_chunks, n_long, stream);
}

extern "C" int llmx_decayed_state_rows(void) { return DS_ROWS; }

extern "C" int llmx_decayed_state_chunks(const float* q, int ldq, const float* k, int ldk, const float* v, int ldv, const float* powers, float* state,
                                         long state_stride, const int* slot_read, const int* slot_write, const int* chunks, int n_chunks,
                                         const int* entry_chunks, int n_long, float* starts, float* out, float out_scale, int H, int D, int V,
                                         int operands, const float* cos_sin, const int* pos, int rot_dims, hipStream_t stream) {
    if (n_chunks <= 0 || n_long <= 0) return 0;
    if (H < 1 || H > 65535 || D < 1 || D > 256 || V < 1 || n_long > 65535 || operands < 0 || operands > 2 || !powers || !starts) return -2;
    if (operands == STATE_OPERANDS_ROTATED && (!cos_sin || !pos || rot_dims < 2 || rot_dims % 2 || rot_dims > D)) return -2;
    const int DR = (D + 15) / 16 * 16, VR = (V + 15) / 16 * 16;
    if ((size_t)H * VR * DR > (size_t)1 << 30) return -2;
    DecayedArgs a{q, k, v, ldq, ldk, ldv, powers, state, state_stride, slot_read, slot_write, chunks, entry_chunks, starts, out, out_scale,
                  H, D, V, DR, VR, StateOperands{cos_sin, pos, rot_dims}};
    llmx_note_launch(LK_DECAYED_STATE_CHUNKS);
    auto at16 = [](const void* p) { return ((uintptr_t)p & 15) == 0; };
    bool vec = at16(q) && at16(k) && at16(v) && ldq % 4 == 0 && ldk % 4 == 0 && ldv % 4 == 0 && D % 4 == 0 && V % 4 == 0;
    if (operands == STATE_OPERANDS_ROTATED) vec = vec && at16(cos_sin) && rot_dims % 8 == 0;
    if (D <= 64) return launch_decayed_kind<4>(a, operands, vec, n_chunks, n_long, stream);
    if (D <= 128) return launch_decayed_kind<8>(a, operands, vec, n_chunks, n_long, stream);
    return launch_decayed_kind<16>(a, operands, vec, n_chunks, n_long, stream);
}
