// What a row takes from the token before it: a bigram row in the embedding, and the token shift of a layer's normed rows.
// The token before a row is the row above it where that belongs to the same entry of the step; for an entry's first row it
// is what the request's state slot kept from the step before.  An entry's last row leaves its own for the next step.
// States are read at `slot_read` and written at `slot_write`; the two are different slots for entries of several rows
// (another workgroup may still read the one while the other is written).
#include "common.h"

// ---------------------------------------------------------------------------
// x[t,:] = table[id[t],:] * scale + bigram[row,:], row = (previous * mul_prev + id[t] * mul_cur) mod buckets, or row number
// `buckets` (the table's last) for a request's first token.  The state is one int a slot: the last token's id + 1, so that
// a cleared slot says "no token yet".  The multipliers come reduced modulo buckets, so the sum fits 64 bits.
template <typename TW>
__global__ void __launch_bounds__(256) embed_bigram_kernel(const TW* __restrict__ table, const TW* __restrict__ bigram, const int* __restrict__ ids,
                                                         int* __restrict__ state, const int* __restrict__ slot_read, const int* __restrict__ slot_write,
                                                         const int* __restrict__ row_entry, const int* __restrict__ entry_rows, float* __restrict__ x,
                                                         int width, float scale, int buckets, long long mul_prev, long long mul_cur) {
    const int t = blockIdx.x;
    const int e = row_entry[t], row0 = entry_rows[2 * e], n = entry_rows[2 * e + 1];
    const int id = ids[t];
    const int before = t > row0 ? ids[t - 1] : state[slot_read[e]] - 1;
    const long long row = before < 0 ? (long long)buckets : ((long long)before * mul_prev + (long long)id * mul_cur) % (long long)buckets;
    const TW* a = table + (size_t)id * width;
    const TW* b = bigram + (size_t)row * width;
    float* out = x + (size_t)t * width;
    for (int i = threadIdx.x; i < width; i += 256) out[i] = ld(a + i) * scale + ld(b + i);
    if (t == row0 + n - 1 && threadIdx.x == 0) state[slot_write[e]] = id + 1;
}

extern "C" int llmx_embed_bigram(const void* table, const void* bigram, int table_dtype, const int* ids, int* state, const int* slot_read,
                                 const int* slot_write, const int* row_entry, const int* entry_rows, float* x, int rows, int width, float scale,
                                 int buckets, long mul_prev, long mul_cur, hipStream_t stream) {
    if (rows <= 0) return 0;
    if (buckets < 1 || mul_prev < 0 || mul_cur < 0 || mul_prev >= buckets || mul_cur >= buckets) return -2;
    llmx_note_launch(LK_EMBED_BIGRAM);
#define LLMX_EB(TW) hipLaunchKernelGGL(embed_bigram_kernel<TW>, dim3(rows), dim3(256), 0, stream, (const TW*)table, (const TW*)bigram, ids, state, \
                                       slot_read, slot_write, row_entry, entry_rows, x, width, scale, buckets, (long long)mul_prev, (long long)mul_cur)
    if (table_dtype == LLMX_F32) LLMX_EB(float);
    else LLMX_EB(bf16_t);
#undef LLMX_EB
    return LLMX_CHECK_LAUNCH();
}

// ---------------------------------------------------------------------------
// Token shift of normed rows: shifted[t] = h[t] + (h[t - 1] - h[t]) * s, element by element, h[-1] the state's row (zeros when
// the request opened).  The state keeps the entry's last h, float32.
struct ShiftArgs {
    const float* x;          // [T, n]: the rows h (token_shift_kernel), or the residual whose norm they are (rmsnorm_shift_kernel)
    const float* norm_w;     // [n]
    float eps;
    const float* shift;      // [n]
    float* state;            // [slots, state_stride], h at its start
    long state_stride;
    const int* slot_read;
    const int* slot_write;
    const int* row_entry;
    const int* entry_rows;
    void* shifted;           // [T, n] in the activation type
    void* out;               // [T, n] in the activation type, or null: h itself
    float* out32;            // [T, n] or null: h unrounded
    int rows, n;
};

__device__ __forceinline__ float shifted_value(float h, float before, float s) { return fmaf(before - h, s, h); }

template <typename TO>
__global__ void __launch_bounds__(256) token_shift_kernel(ShiftArgs a) {
    const int t = blockIdx.x;
    const int e = a.row_entry[t], row0 = a.entry_rows[2 * e], rows = a.entry_rows[2 * e + 1];
    const float* row = a.x + (size_t)t * a.n;
    const float* above = t > row0 ? row - a.n : a.state + (size_t)a.slot_read[e] * a.state_stride;
    float* keep = t == row0 + rows - 1 ? a.state + (size_t)a.slot_write[e] * a.state_stride : nullptr;
    for (int i = threadIdx.x; i < a.n; i += 256) {
        const float h = row[i];
        st((TO*)a.shifted + (size_t)t * a.n + i, shifted_value(h, above[i], a.shift[i]));
        if (keep) keep[i] = h;
    }
}

// The norm and the shift in one launch: h = x * (r * w) with the bits of the norm kernel (1,024 threads a row, the sum in its
// order).  A workgroup takes ROWS consecutive rows; the row above its first is normed again, from its own sum, with the bits
// its own workgroup gives it (or comes from the state, normed already).  KEPT > 0: rows of at most 1,024 * KEPT values stay in
// registers, all asked for before the first sum.
#define SHIFT_THREADS 1024
template <typename TO, int KEPT, int ROWS>
__global__ void __launch_bounds__(SHIFT_THREADS) rmsnorm_shift_kernel(ShiftArgs a) {
    constexpr int WAVES = SHIFT_THREADS / 64;
    __shared__ float scratch[ROWS + 1][WAVES];
    const int n = a.n, t0 = blockIdx.x * ROWS, last = min(t0 + ROWS, a.rows) - 1;
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    // row u of the workgroup is the step's row t0 - 1 + u: u 0 is the row above the first
    auto source = [&](int u) -> const float* {
        const int t = min(t0 - 1 + u, last);
        if (u == 0) {
            const int e = a.row_entry[t0];
            if (t0 == a.entry_rows[2 * e]) return a.state + (size_t)a.slot_read[e] * a.state_stride;
        }
        return a.x + (size_t)t * n;
    };
    constexpr int K = KEPT > 0 ? KEPT : 1;
    float v[ROWS + 1][K], w[K], s[K];
    if (KEPT > 0) {
#pragma unroll
        for (int u = 0; u <= ROWS; ++u) {
            const float* row = source(u);
#pragma unroll
            for (int k = 0; k < K; ++k) {
                const int i = threadIdx.x + k * SHIFT_THREADS;
                v[u][k] = i < n ? row[i] : 0.0f;
            }
        }
#pragma unroll
        for (int k = 0; k < K; ++k) {
            const int i = threadIdx.x + k * SHIFT_THREADS;
            w[k] = i < n ? a.norm_w[i] : 0.0f;
            s[k] = i < n ? a.shift[i] : 0.0f;
        }
    }
#pragma unroll
    for (int u = 0; u <= ROWS; ++u) {
        float sq = 0.0f;
        if (KEPT > 0) {
#pragma unroll
            for (int k = 0; k < K; ++k) sq = fmaf(v[u][k], v[u][k], sq);
        } else {
            sq = strided_squares<SHIFT_THREADS>(source(u), n);
        }
        sq = wave_sum(sq);
        if (lane == 0) scratch[u][wave] = sq;
    }
    __syncthreads();
    float r[ROWS + 1];
#pragma unroll
    for (int u = 0; u <= ROWS; ++u) {
        float sum = scratch[u][0];
#pragma unroll
        for (int k = 1; k < WAVES; ++k) sum += scratch[u][k];
        r[u] = 1.0f / sqrtf(sum / (float)n + a.eps);
    }
#pragma unroll
    for (int u = 1; u <= ROWS; ++u) {
        const int t = t0 - 1 + u;
        if (t > last) break;
        const int e = a.row_entry[t], row0 = a.entry_rows[2 * e], rows = a.entry_rows[2 * e + 1];
        const bool inside = t > row0;
        const float* opened = a.state + (size_t)a.slot_read[e] * a.state_stride;     // read where an entry begins
        float* keep = t == row0 + rows - 1 ? a.state + (size_t)a.slot_write[e] * a.state_stride : nullptr;
        auto finish = [&](int i, float x, float y, float wi, float si) {
            const float h = x * (r[u] * wi);
            const float before = inside ? y * (r[u - 1] * wi) : y;
            const size_t at = (size_t)t * n + i;
            st((TO*)a.shifted + at, shifted_value(h, before, si));
            if (a.out) st((TO*)a.out + at, h);
            if (a.out32) a.out32[at] = h;
            if (keep) keep[i] = h;
        };
        if (KEPT > 0) {
#pragma unroll
            for (int k = 0; k < K; ++k) {
                const int i = threadIdx.x + k * SHIFT_THREADS;
                if (i < n) finish(i, v[u][k], inside || u == 1 ? v[u - 1][k] : opened[i], w[k], s[k]);
            }
        } else {
            const float* row = a.x + (size_t)t * n;
            const float* above = inside ? row - n : opened;
            for (int i = threadIdx.x; i < n; i += SHIFT_THREADS) finish(i, row[i], above[i], a.norm_w[i], a.shift[i]);
        }
    }
}

// norm_w null: x holds the rows h themselves (and out, out32 are not written).
extern "C" int llmx_token_shift(const float* x, const float* norm_w, float eps, const float* shift, float* state, long state_stride,
                                const int* slot_read, const int* slot_write, const int* row_entry, const int* entry_rows, void* shifted, void* out,
                                float* out32, int out_dtype, int rows, int n, hipStream_t stream) {
    if (rows <= 0 || n <= 0) return 0;
    if (state_stride < n || !shift || !state || !shifted) return -2;
    ShiftArgs a{x, norm_w, eps, shift, state, state_stride, slot_read, slot_write, row_entry, entry_rows, shifted, out, out32, rows, n};
    if (!norm_w) {
        llmx_note_launch(LK_TOKEN_SHIFT);
        if (out_dtype == LLMX_F32) hipLaunchKernelGGL(token_shift_kernel<float>, dim3(rows), dim3(256), 0, stream, a);
        else hipLaunchKernelGGL(token_shift_kernel<bf16_t>, dim3(rows), dim3(256), 0, stream, a);
        return LLMX_CHECK_LAUNCH();
    }
    llmx_note_launch(LK_RMSNORM_SHIFT);
#define LLMX_RS(KEPT, ROWS) \
    do { \
        const dim3 grid((unsigned)((rows + ROWS - 1) / ROWS)); \
        if (out_dtype == LLMX_F32) hipLaunchKernelGGL((rmsnorm_shift_kernel<float, KEPT, ROWS>), grid, dim3(SHIFT_THREADS), 0, stream, a); \
        else hipLaunchKernelGGL((rmsnorm_shift_kernel<bf16_t, KEPT, ROWS>), grid, dim3(SHIFT_THREADS), 0, stream, a); \
    } while (0)
    // steps of many rows: a workgroup takes four rows where their values fit its registers
    if (n <= SHIFT_THREADS * 2) {
        if (rows >= 1024) LLMX_RS(2, 4);
        else LLMX_RS(2, 1);
    } else if (n <= SHIFT_THREADS * 4) {
        if (rows >= 1024) LLMX_RS(4, 4);
        else LLMX_RS(4, 1);
    } else if (n <= SHIFT_THREADS * 8) {
        LLMX_RS(8, 1);
    } else {
        LLMX_RS(0, 1);
    }
#undef LLMX_RS
    return LLMX_CHECK_LAUNCH();
}
