// The gated delta rule with one decay g_t a head and token,
//     S <- g_t S,   u_t = beta_t (v_t - S^T k_t),   S <- S + k_t u_t^T,   o_t = S^T q_t,
// for long runs of rows, chunk by chunk on the float32 matrix instruction (short runs: state_scan of linear_state.hip; the two
// differ by rounding).  With i, j counting a chunk's rows from 0, S the state before it and L_i = sum_(m <= i) log g_m, the
// corrections u of a chunk solve a unit lower triangular system:
//     (I + A) U = B V - B e^L K S,    A_ij = beta_i e^(L_i - L_j) k_i . k_j  (j < i),   B = diag(beta)
// so with T = (I + A)^-1,  U = T B V - (T B e^L K) S = U0 - W S, and then
//     o_i = e^L_i S^T q_i + sum_(j <= i) e^(L_i - L_j) (q_i . k_j) u_j,     S <- e^L_last S + sum_j e^(L_last - L_j) k_j u_j^T.
// Every exponential is of a sum of logarithms that are at most 0; the sums are formed in float64, so a difference of two of them
// is as exact as its terms.  Three launches:
//   solve   a workgroup a (chunk, head): A, T (16 x 16 blocks on the diagonal by substitution, the blocks below them as products),
//           W, U0 and the chunk's decays;
//   states  a workgroup a (request, head, 16 value channels): walks the request's chunks in order, its state in registers (a wave
//           16 key channels): leaves the state before each chunk in `starts`, turns U0 into U, writes the last state to the slot;
//   rows    a workgroup a (chunk, head): the read-out (state_chunks.h).
// Everything is float32 but the sums of logarithms.
#include "state_chunks.h"

#define DC_LDT 68            // floats of a row of A (and T) in LDS

struct DeltaChunkArgs {
    const float* q;          // unit vectors: q, k [T, H / share * D], v [T, H * V]
    const float* k;
    const float* v;
    int ldq, ldk, ldv;
    const float* beta;       // [T, H]
    const float* log_decay;  // [T, H]: log g
    float* state;            // S at the slot's start, in the scan's tiles: [H, ceil(V / 8), D, 8]
    long state_stride;
    const int* slot_read;
    const int* slot_write;
    const int* chunks;       // [n_chunks, 4]: entry, first row, rows, -
    const int* entry_chunks; // [n_long, 4]: entry, first chunk, chunks, -
    float* W;                // [chunk][head][64][DR]
    float* U;                // [chunk][head][64][VR]: U0, then U
    float* decays;           // [chunk][head][64]: e^(L_last - L_j)
    float* keep;             // [chunk][head]: e^L_last
    float* starts;           // [chunk][head][VR][DR]
    float* out;              // [T, H * V]
    float out_scale;
    int H, share, D, V, DR, VR;
    const float* tail_src;   // [T, tail_ld]: rows whose last taps - 1 become the request's new tail at tail_off of its slot (null: none)
    int tail_ld, tail_C, taps, tail_off;
    const int* entry_rows;
};

__device__ __forceinline__ ChunkRows delta_chunk_rows(const DeltaChunkArgs& a, bool corrected) {
    const int* chunk = a.chunks + 4 * (size_t)blockIdx.x;
    const int row0 = chunk[1], n = chunk[2], h = blockIdx.y, hk = h / a.share;
    const size_t at = (size_t)blockIdx.x * a.H + h;
    return ChunkRows{a.q + (size_t)row0 * a.ldq + (size_t)hk * a.D, a.k + (size_t)row0 * a.ldk + (size_t)hk * a.D,
                     corrected ? a.U + at * DS_ROWS * a.VR : a.v + (size_t)row0 * a.ldv + (size_t)h * a.V, a.ldq, a.ldk, corrected ? a.VR : a.ldv,
                     row0, n, a.D, a.V, a.DR, a.VR, a.starts + at * a.VR * a.DR, a.out + (size_t)row0 * a.H * a.V + (size_t)h * a.V, a.H * a.V,
                     a.out_scale, StateOperands{nullptr, nullptr, 0}};
}

// L of the chunk's 64 rows by the first wave: an inclusive sum in float64 (rows past the chunk's add 0).
__device__ __forceinline__ double chunk_log_sums(const DeltaChunkArgs& a, int row0, int n, int h, int lane) {
    double s = lane < n ? (double)a.log_decay[(size_t)(row0 + lane) * a.H + h] : 0.0;
#pragma unroll
    for (int d = 1; d < 64; d <<= 1) {
        const double before = __shfl_up(s, d, 64);
        if (lane >= d) s += before;
    }
    return s;
}

// NU: a head's key channels in tiles of 16, padded
template <int NU, bool VEC>
__global__ void __launch_bounds__(256) delta_chunk_solve_kernel(DeltaChunkArgs a) {
    constexpr int DP = 16 * NU, LDK = DP + 4, LDV = 64 + 4;
    extern __shared__ __align__(16) float lds[];
    float* ks = lds;                               // [64][LDK]
    float* vs = ks + DS_ROWS * LDK;                // [64][LDV]
    float* as = vs + DS_ROWS * LDV;                // [64][DC_LDT]: A, then T
    float* beta = as + DS_ROWS * DC_LDT;           // [64]
    float* row_w = beta + DS_ROWS;                 // [64]: beta e^L
    double* L = reinterpret_cast<double*>(row_w + DS_ROWS);    // [64]
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, c = lane & 15, g = lane >> 4;
    const ChunkRows rows = delta_chunk_rows(a, false);
    const int n = rows.n, h = blockIdx.y;
    const size_t at = (size_t)blockIdx.x * a.H + h;
    if (wave == 0) {
        const double l = chunk_log_sums(a, rows.row0, n, h, lane);
        const float b = lane < n ? a.beta[(size_t)(rows.row0 + lane) * a.H + h] : 0.0f;
        const double last = __shfl(l, 63, 64);
        L[lane] = l;
        beta[lane] = b;
        row_w[lane] = b * expf((float)l);
        a.decays[at * DS_ROWS + lane] = expf((float)(last - l));
        if (lane == 0) a.keep[at] = expf((float)last);
    }
    stage_keys<NU, STATE_OPERANDS_PLAIN, VEC, LDK>(rows, ks);
    __syncthreads();
    // A: key row 16 t + 4 g + e against row 16 wave + c, t up to the wave's own tile
    {
        f32x4_t s[4];
#pragma unroll
        for (int t = 0; t < 4; ++t) s[t] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
        const float* own = ks + (16 * wave + c) * LDK + 4 * g;
#pragma unroll
        for (int u = 0; u < NU; ++u) {
            const f32x4_t q = *reinterpret_cast<const f32x4_t*>(own + 16 * u);
#pragma unroll
            for (int t = 0; t < 4; ++t) {
                if (t <= wave) {
                    const f32x4_t kf = *reinterpret_cast<const f32x4_t*>(ks + (16 * t + c) * LDK + 16 * u + 4 * g);
#pragma unroll
                    for (int e = 0; e < 4; ++e) s[t] = mfma4(kf[e], q[e], s[t]);
                }
            }
        }
        const int i = 16 * wave + c;
        const double li = L[i];
        const float bi = beta[i];
#pragma unroll
        for (int t = 0; t < 4; ++t) {
            if (t <= wave) {
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const int j = 16 * t + 4 * g + e;
                    s[t][e] = j < i ? s[t][e] * (bi * expf((float)(li - L[j]))) : 0.0f;
                }
                *reinterpret_cast<f32x4_t*>(as + i * DC_LDT + 16 * t + 4 * g) = s[t];
            }
        }
    }
    __syncthreads();
    // the inverse of the wave's block on the diagonal, a column a lane (the four groups of lanes alike), by forward substitution
    f32x4_t t_own;           // rows 4 g + e of column c
    {
        float x[16];
        const float* block = as + 16 * wave * DC_LDT + 16 * wave;
#pragma unroll
        for (int r = 0; r < 16; ++r) {
            float sum = r == c ? 1.0f : 0.0f;
#pragma unroll
            for (int s4 = 0; s4 < (r + 3) / 4; ++s4) {
                const f32x4_t m = *reinterpret_cast<const f32x4_t*>(block + r * DC_LDT + 4 * s4);
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (4 * s4 + e < r) sum = fmaf(-m[e], x[4 * s4 + e], sum);
            }
            x[r] = sum;
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) t_own[e] = g == 0 ? x[e] : g == 1 ? x[4 + e] : g == 2 ? x[8 + e] : x[12 + e];
    }
    // in place of A's block, which nobody else reads
#pragma unroll
    for (int e = 0; e < 4; ++e) as[(16 * wave + 4 * g + e) * DC_LDT + 16 * wave + c] = t_own[e];
    __syncthreads();
    // the blocks below: wave j forms column j, T_ij = -T_ii sum_(j <= m < i) A_im T_mj
    f32x4_t col[4];
    col[0] = t_own;          // col[m - wave]
#pragma unroll
    for (int step = 1; step < 4; ++step) {
        const int i = wave + step;
        if (i < 4) {
            f32x4_t p = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
            for (int m = 0; m < step; ++m) {
                const f32x4_t x = *reinterpret_cast<const f32x4_t*>(as + (16 * i + c) * DC_LDT + 16 * (wave + m) + 4 * g);
#pragma unroll
                for (int e = 0; e < 4; ++e) p = mfma4(x[e], col[m][e], p);
            }
            const f32x4_t d = *reinterpret_cast<const f32x4_t*>(as + (16 * i + c) * DC_LDT + 16 * i + 4 * g);
            f32x4_t r = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
            for (int e = 0; e < 4; ++e) r = mfma4(-d[e], p[e], r);
            col[step] = r;
        }
    }
    __syncthreads();         // A has been read by every wave
#pragma unroll
    for (int step = 1; step < 4; ++step)
        if (wave + step < 4) {
#pragma unroll
            for (int e = 0; e < 4; ++e) as[(16 * (wave + step) + 4 * g + e) * DC_LDT + 16 * wave + c] = col[step][e];
        }
    stage_values<STATE_OPERANDS_PLAIN, VEC, LDV>(rows, 0, vs, [&](int j) { return beta[j]; });
    __syncthreads();
    // T's rows as the products' first operand: tf[i (i + 1) / 2 + m] row 16 i + c, columns 16 m + 4 g + e
    f32x4_t tf[10];
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int m = 0; m <= i; ++m) tf[i * (i + 1) / 2 + m] = *reinterpret_cast<const f32x4_t*>(as + (16 * i + c) * DC_LDT + 16 * m + 4 * g);
    float rw[4][4];
#pragma unroll
    for (int m = 0; m < 4; ++m)
#pragma unroll
        for (int e = 0; e < 4; ++e) rw[m][e] = row_w[16 * m + 4 * g + e];
    // W = T (beta e^L K), the waves taking turns at tiles of 16 key channels
    float* w_to = a.W + at * DS_ROWS * a.DR;
#pragma unroll
    for (int u0 = 0; u0 < NU; u0 += 4) {
        const int u = u0 + wave;
        if (16 * u < a.DR) {
            f32x4_t acc[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) acc[i] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
            for (int m = 0; m < 4; ++m)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const float b = ks[(16 * m + 4 * g + e) * LDK + 16 * u + c] * rw[m][e];
#pragma unroll
                    for (int i = m; i < 4; ++i) acc[i] = mfma4(tf[i * (i + 1) / 2 + m][e], b, acc[i]);
                }
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int e = 0; e < 4; ++e) w_to[(size_t)(16 * i + 4 * g + e) * a.DR + 16 * u + c] = acc[i][e];
        }
    }
    // U0 = T (beta V), 64 value channels at a time
    float* u_to = a.U + at * DS_ROWS * a.VR;
    for (int v0 = 0; v0 < a.VR; v0 += 64) {
        if (v0 > 0) {
            __syncthreads();
            stage_values<STATE_OPERANDS_PLAIN, VEC, LDV>(rows, v0, vs, [&](int j) { return beta[j]; });
            __syncthreads();
        }
        if (v0 + 16 * wave < a.VR) {
            f32x4_t acc[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) acc[i] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
            for (int m = 0; m < 4; ++m)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const float b = vs[(16 * m + 4 * g + e) * LDV + 16 * wave + c];
#pragma unroll
                    for (int i = m; i < 4; ++i) acc[i] = mfma4(tf[i * (i + 1) / 2 + m][e], b, acc[i]);
                }
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int e = 0; e < 4; ++e) u_to[(size_t)(16 * i + 4 * g + e) * a.VR + v0 + 16 * wave + c] = acc[i][e];
        }
    }
}

// Grid (H * value tiles, long requests), a wave for every 16 key channels.  The operands of the chunks to
// come are asked for while one is worked on.
template <int NU>
__global__ void __launch_bounds__(64 * NU) delta_chunk_states_kernel(DeltaChunkArgs a) {
    constexpr int NT = 64 * NU, EL = 1024 / NT, LDU = 20;      // EL: values of the chunk's U (64 x 16) a thread adds up
    __shared__ __align__(16) float part[NU][1024];
    __shared__ float us[DS_ROWS * LDU];
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, c = lane & 15, g = lane >> 4;
    const int* ec = a.entry_chunks + 4 * (size_t)blockIdx.y;
    const int entry = ec[0], c0 = ec[1], nc = ec[2];
    const int h = blockIdx.x % a.H, vt = blockIdx.x / a.H;
    const int row0 = a.entry_rows[2 * entry], rows = a.entry_rows[2 * entry + 1];      // its chunks' rows follow each other
    const size_t slot_r = (size_t)a.slot_read[entry] * a.state_stride, slot_w = (size_t)a.slot_write[entry] * a.state_stride;

    if (a.taps > 1) {       // the request's workgroups share the tail's channels out among themselves
        const float* old = a.state + slot_r + a.tail_off;
        float* fresh = a.state + slot_w + a.tail_off;
        const int per = (a.tail_C + (int)gridDim.x - 1) / (int)gridDim.x, end = min(a.tail_C, ((int)blockIdx.x + 1) * per);
        for (int ch = (int)blockIdx.x * per + tid; ch < end; ch += NT)
            for (int p = 0; p < a.taps - 1; ++p) {          // ascending: in place, a value is read before its place is written
                const int idx = rows - (a.taps - 1) + p;
                fresh[(size_t)p * a.tail_C + ch] = idx >= 0 ? a.tail_src[(size_t)(row0 + idx) * a.tail_ld + ch] : old[(size_t)(rows + p) * a.tail_C + ch];
            }
    }

    const bool real = 16 * wave < a.DR;        // a wave past the key channels adds zeros
    const int v = 16 * vt + c, tiles = (a.V + 7) / 8;
    const size_t tile_at = ((size_t)h * tiles + v / 8) * a.D * 8 + v % 8;
    f32x4_t S;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        const int d = 16 * wave + 4 * g + e;
        const bool in = v < a.V && d < a.D;
        const float x = a.state[slot_r + (in ? tile_at + (size_t)d * 8 : 0)];
        S[e] = in ? x : 0.0f;
    }
    struct Operands {
        f32x4_t w[4];        // W: row 16 i + c, key channels 16 wave + 4 g + e
        float k[16];         // k: row 16 s + 4 g + e, key channel 16 wave + c
        float u0[EL], decay[EL];
        float keep;
    };
    const int first = EL * tid;                             // the thread's values: row and column from its place in a tile's lanes
    const int u_row0 = 16 * (first >> 8) + 4 * ((first & 255) >> 6), u_col = ((first & 255) >> 2) & 15, u_e0 = first & 3;
    const int kd = min(16 * wave + c, a.D - 1), wd = real ? 16 * wave + 4 * g : 0;
    // a thread's places within a chunk's operands, in bytes from a base that is the same for every thread
    const uint32_t w_at = 4u * (uint32_t)(c * a.DR + wd), k_at = 4u * (uint32_t)(4 * g * a.ldk + kd);
    const uint32_t u_at = 4u * (uint32_t)((u_row0 + u_e0) * a.VR + 16 * vt + u_col), d_at = 4u * (uint32_t)(u_row0 + u_e0);
    const uint32_t start_at = 4u * (uint32_t)((16 * vt + c) * a.DR + 16 * wave + 4 * g);
    auto fetch = [&](Operands& x, int ch) {
        const size_t at = (size_t)ch * a.H + h;
        const float* W = a.W + at * DS_ROWS * a.DR;
#pragma unroll
        for (int i = 0; i < 4; ++i) x.w[i] = *reinterpret_cast<const f32x4_t*>(reinterpret_cast<const char*>(W + (size_t)(16 * i) * a.DR) + w_at);
        const int ahead = (ch - c0) * DS_ROWS, n = min(DS_ROWS, rows - ahead);
        const float* kp = a.k + (size_t)(row0 + ahead) * a.ldk + (size_t)(h / a.share) * a.D;
        if (n == DS_ROWS) {
#pragma unroll
            for (int s = 0; s < 4; ++s)
#pragma unroll
                for (int e = 0; e < 4; ++e) x.k[4 * s + e] = *reinterpret_cast<const float*>(reinterpret_cast<const char*>(kp + (size_t)(16 * s + e) * a.ldk) + k_at);
        } else {
#pragma unroll
            for (int s = 0; s < 4; ++s)
#pragma unroll
                for (int e = 0; e < 4; ++e) x.k[4 * s + e] = kp[(size_t)min(16 * s + 4 * g + e, n - 1) * a.ldk + kd];
        }
        const float* U = a.U + at * DS_ROWS * a.VR;
        const float* decays = a.decays + at * DS_ROWS;
#pragma unroll
        for (int y = 0; y < EL; ++y) {
            x.u0[y] = *reinterpret_cast<const float*>(reinterpret_cast<const char*>(U + (size_t)y * a.VR) + u_at);
            x.decay[y] = *reinterpret_cast<const float*>(reinterpret_cast<const char*>(decays + y) + d_at);
        }
        x.keep = a.keep[at];
    };
    auto work = [&](const Operands& x, int ch) {
        const size_t at = (size_t)ch * a.H + h;
        if (real) *reinterpret_cast<f32x4_t*>(reinterpret_cast<char*>(a.starts + at * a.VR * a.DR) + start_at) = S;
        f32x4_t p[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) p[i] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
        for (int e = 0; e < 4; ++e)
#pragma unroll
            for (int i = 0; i < 4; ++i) p[i] = mfma4(x.w[i][e], S[e], p[i]);
#pragma unroll
        for (int i = 0; i < 4; ++i) *reinterpret_cast<f32x4_t*>(&part[wave][i * 256 + lane * 4]) = p[i];
        __syncthreads();
#pragma unroll
        for (int y = 0; y < EL; ++y) {
            float sum = part[0][first + y];
#pragma unroll
            for (int w = 1; w < NU; ++w) sum += part[w][first + y];
            const float u = x.u0[y] - sum;
            const int row = u_row0 + u_e0 + y;
            *reinterpret_cast<float*>(reinterpret_cast<char*>(a.U + (at * DS_ROWS + y) * a.VR) + u_at) = u;
            us[row * LDU + u_col] = u * x.decay[y];
        }
        __syncthreads();
        float b[16];
#pragma unroll
        for (int s = 0; s < 4; ++s)
#pragma unroll
            for (int e = 0; e < 4; ++e) b[4 * s + e] = us[(16 * s + 4 * g + e) * LDU + c];
        __builtin_amdgcn_sched_barrier(0);      // all of them asked for before the first product waits for one
        f32x4_t add[2];
        add[0] = f32x4_t{S[0] * x.keep, S[1] * x.keep, S[2] * x.keep, S[3] * x.keep};
        add[1] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
        for (int s = 0; s < 4; ++s)
#pragma unroll
            for (int e = 0; e < 4; ++e) add[e & 1] = mfma4(x.k[4 * s + e], b[4 * s + e], add[e & 1]);
#pragma unroll
        for (int e = 0; e < 4; ++e) S[e] = 16 * wave + 4 * g + e < a.D ? add[0][e] + add[1][e] : 0.0f;
    };
    // sets of operands that take turns: the next AHEAD chunks' are on their way while one is worked on (past the end the last again)
    constexpr int AHEAD = NU > 8 ? 1 : 2;
    Operands ring[AHEAD + 1];
#pragma unroll
    for (int u = 0; u < AHEAD; ++u) fetch(ring[u], c0 + min(u, nc - 1));
    for (int i = 0; i < nc; i += AHEAD + 1) {
#pragma unroll
        for (int u = 0; u <= AHEAD; ++u) {
            if (i + u < nc) {
                fetch(ring[(u + AHEAD) % (AHEAD + 1)], c0 + min(i + u + AHEAD, nc - 1));
                work(ring[u], c0 + i + u);
            }
        }
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        const int d = 16 * wave + 4 * g + e;
        if (v < a.V && d < a.D) a.state[slot_w + tile_at + (size_t)d * 8] = S[e];
    }
}

// The decays of a chunk's rows from their sums of logarithms.
struct LogDecay {
    const double* L;         // [64] in LDS
    __device__ __forceinline__ float between(int i, int j) const { return expf((float)(L[i] - L[j])); }
    __device__ __forceinline__ float upto(int i) const { return expf((float)L[i]); }
};

template <int NU, bool VEC>
__global__ void __launch_bounds__(256) delta_chunk_rows_kernel(DeltaChunkArgs a) {
    extern __shared__ __align__(16) float lds[];
    double* L = reinterpret_cast<double*>(lds + state_rows_lds(NU));
    const ChunkRows rows = delta_chunk_rows(a, true);
    if (threadIdx.x < 64) L[threadIdx.x] = chunk_log_sums(a, rows.row0, rows.n, blockIdx.y, threadIdx.x);
    state_rows_read<NU, STATE_OPERANDS_PLAIN, VEC>(rows, LogDecay{L}, lds);
}

template <int NU, bool VEC>
static int launch_delta_chunks(const DeltaChunkArgs& a, int n_chunks, int n_long, hipStream_t stream) {
    constexpr size_t lds_solve = sizeof(float) * DS_ROWS * (16 * NU + 4 + 64 + 4 + DC_LDT + 2) + sizeof(double) * DS_ROWS;
    constexpr size_t lds_rows = sizeof(float) * state_rows_lds(NU) + sizeof(double) * DS_ROWS;
    static bool raised = false;
    if (!raised) {
        if (hipFuncSetAttribute((const void*)delta_chunk_solve_kernel<NU, VEC>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024) != hipSuccess) return -1;
        if (hipFuncSetAttribute((const void*)delta_chunk_rows_kernel<NU, VEC>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024) != hipSuccess) return -1;
        raised = true;
    }
    hipLaunchKernelGGL((delta_chunk_solve_kernel<NU, VEC>), dim3(n_chunks, a.H), dim3(256), lds_solve, stream, a);
    hipLaunchKernelGGL(delta_chunk_states_kernel<NU>, dim3(a.H * (a.VR / 16), n_long), dim3(64 * NU), 0, stream, a);
    hipLaunchKernelGGL((delta_chunk_rows_kernel<NU, VEC>), dim3(n_chunks, a.H), dim3(256), lds_rows, stream, a);
    return LLMX_CHECK_LAUNCH();
}

extern "C" int llmx_delta_chunks(const float* q, int ldq, const float* k, int ldk, const float* v, int ldv, const float* beta, const float* log_decay,
                                 float* state, long state_stride, const int* slot_read, const int* slot_write, const int* entry_rows, const int* chunks,
                                 int n_chunks, const int* entry_chunks, int n_long, float* W, float* U, float* decays, float* keep, float* starts,
                                 float* out, float out_scale, int H, int share, int D, int V, const float* tail_src, int tail_ld, int tail_C, int taps,
                                 int tail_off, hipStream_t stream) {
    if (n_chunks <= 0 || n_long <= 0) return 0;
    if (H < 1 || H > 65535 || share < 1 || H % share || D < 1 || D > 256 || V < 1 || n_long > 65535 || (taps > 1 && !tail_src)) return -2;
    const int DR = (D + 15) / 16 * 16, VR = (V + 15) / 16 * 16;
    if ((size_t)H * VR * DR > (size_t)1 << 30 || (size_t)VR * DR > (size_t)1 << 28 || (size_t)ldk > (size_t)1 << 24) return -2;
    DeltaChunkArgs a{q, k, v, ldq, ldk, ldv, beta, log_decay, state, state_stride, slot_read, slot_write, chunks, entry_chunks, W, U, decays, keep,
                     starts, out, out_scale, H, share, D, V, DR, VR, tail_src, tail_ld, tail_C, taps, tail_off, entry_rows};
    llmx_note_launch(LK_DELTA_CHUNKS);
    auto at16 = [](const void* p) { return ((uintptr_t)p & 15) == 0; };
    const bool vec = at16(q) && at16(k) && at16(v) && ldq % 4 == 0 && ldk % 4 == 0 && ldv % 4 == 0 && D % 4 == 0 && V % 4 == 0;
#define LLMX_DC(NU) (vec ? launch_delta_chunks<NU, true>(a, n_chunks, n_long, stream) : launch_delta_chunks<NU, false>(a, n_chunks, n_long, stream))
    if (D <= 64) return LLMX_DC(4);
    if (D <= 128) return LLMX_DC(8);
    return LLMX_DC(16);
#undef LLMX_DC
}
