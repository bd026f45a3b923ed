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
    int n;
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
// order); the row above is normed again by the same workgroup, from its own sum, with the bits its own workgroup gives it.
// Rows of at most 1,024 * SHIFT_KEPT values stay in registers, both asked for before the first sum.
#define SHIFT_THREADS 1024
#define SHIFT_KEPT 8
template <typename TO, bool KEPT>
__global__ void __launch_bounds__(SHIFT_THREADS) rmsnorm_shift_kernel(ShiftArgs a) {
    __shared__ float scratch[2][SHIFT_THREADS / 64];
    const int t = blockIdx.x, n = a.n;
    const int e = a.row_entry[t], row0 = a.entry_rows[2 * e], rows = a.entry_rows[2 * e + 1];
    const bool inside = t > row0;
    const float* row = a.x + (size_t)t * n;
    const float* above = inside ? row - n : a.state + (size_t)a.slot_read[e] * a.state_stride;
    float v[SHIFT_KEPT], u[SHIFT_KEPT], w[SHIFT_KEPT], s[SHIFT_KEPT];
    float sq = 0.0f, sq_above = 0.0f;
    if (KEPT) {
#pragma unroll
        for (int k = 0; k < SHIFT_KEPT; ++k) {
            const int i = threadIdx.x + k * SHIFT_THREADS;
            v[k] = i < n ? row[i] : 0.0f;
            u[k] = i < n ? above[i] : 0.0f;
            w[k] = i < n ? a.norm_w[i] : 0.0f;
            s[k] = i < n ? a.shift[i] : 0.0f;
        }
#pragma unroll
        for (int k = 0; k < SHIFT_KEPT; ++k) {
            sq = fmaf(v[k], v[k], sq);
            sq_above = fmaf(u[k], u[k], sq_above);
        }
    } else {
        sq = strided_squares<SHIFT_THREADS>(row, n);
        if (inside) sq_above = strided_squares<SHIFT_THREADS>(above, n);
    }
    // both sums with one barrier: a butterfly a wave, the waves in order
    sq = wave_sum(sq);
    sq_above = wave_sum(sq_above);
    if ((threadIdx.x & 63) == 0) {
        scratch[0][threadIdx.x >> 6] = sq;
        scratch[1][threadIdx.x >> 6] = sq_above;
    }
    __syncthreads();
    float sum = scratch[0][0], sum_above = scratch[1][0];
#pragma unroll
    for (int k = 1; k < SHIFT_THREADS / 64; ++k) {
        sum += scratch[0][k];
        sum_above += scratch[1][k];
    }
    const float r = 1.0f / sqrtf(sum / (float)n + a.eps);
    const float r_above = 1.0f / sqrtf(sum_above / (float)n + a.eps);
    float* keep = t == row0 + rows - 1 ? a.state + (size_t)a.slot_write[e] * a.state_stride : nullptr;
    auto finish = [&](int i, float x, float y, float wi, float si) {
        const float h = x * (r * wi);
        const float before = inside ? y * (r_above * wi) : y;        // a state's row is normed already
        const size_t at = (size_t)t * n + i;
        st((TO*)a.shifted + at, shifted_value(h, before, si));
        if (a.out) st((TO*)a.out + at, h);
        if (a.out32) a.out32[at] = h;
        if (keep) keep[i] = h;
    };
    if (KEPT) {
#pragma unroll
        for (int k = 0; k < SHIFT_KEPT; ++k) {
            const int i = threadIdx.x + k * SHIFT_THREADS;
            if (i < n) finish(i, v[k], u[k], w[k], s[k]);
        }
    } else {
        for (int i = threadIdx.x; i < n; i += SHIFT_THREADS) finish(i, row[i], above[i], a.norm_w[i], a.shift[i]);
    }
}

// norm_w null: x holds the rows h themselves (and out, out32 are not written).
extern "C" int llmx_token_shift(const float* x, const float* norm_w, float eps, const float* shift, float* state, long state_stride,
                                const int* slot_read, const int* slot_write, const int* row_entry, const int* entry_rows, void* shifted, void* out,
                                float* out32, int out_dtype, int rows, int n, hipStream_t stream) {
    if (rows <= 0 || n <= 0) return 0;
    if (state_stride < n || !shift || !state || !shifted) return -2;
    ShiftArgs a{x, norm_w, eps, shift, state, state_stride, slot_read, slot_write, row_entry, entry_rows, shifted, out, out32, n};
    if (!norm_w) {
        llmx_note_launch(LK_TOKEN_SHIFT);
        if (out_dtype == LLMX_F32) hipLaunchKernelGGL(token_shift_kernel<float>, dim3(rows), dim3(256), 0, stream, a);
        else hipLaunchKernelGGL(token_shift_kernel<bf16_t>, dim3(rows), dim3(256), 0, stream, a);
        return LLMX_CHECK_LAUNCH();
    }
    llmx_note_launch(LK_RMSNORM_SHIFT);
    const bool kept = n <= SHIFT_THREADS * SHIFT_KEPT;
#define LLMX_RS(TO, KEPT) hipLaunchKernelGGL((rmsnorm_shift_kernel<TO, KEPT>), dim3(rows), dim3(SHIFT_THREADS), 0, stream, a)
    if (out_dtype == LLMX_F32) {
        if (kept) LLMX_RS(float, true);
        else LLMX_RS(float, false);
    } else {
        if (kept) LLMX_RS(bf16_t, true);
        else LLMX_RS(bf16_t, false);
    }
#undef LLMX_RS
    return LLMX_CHECK_LAUNCH();
}
