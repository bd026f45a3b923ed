// Layer norm with a weight and an optional bias, and the element-wise steps of layers that norm a sublayer's result before it
// joins the residual: y = (x - mean) / sqrt(var + eps) * w (+ b), var the mean of the squared deviations.  Everything is float32
// arithmetic on float32 rows; only what a product reads next is stored in the activation type.
// A row's sums are formed by 256 threads: thread v adds elements v, v + 256, ... in this order, a wave adds its threads' sums with
// wave_sum, and the four waves' sums are added in wave order.  Norms with a bias whose rows are a multiple of 4 long deal the elements
// out by fours instead (4v .. 4v + 3, then those 1,024 further on, ...), so that a thread reads and writes 16 bytes at a time.  Either
// way a row's bits depend on its length and its norm only.
#include "common.h"

#define LN_THREADS 256
#define LN_QUADS 4      // groups of four values a thread keeps in registers: rows of at most 4,096 values are read once

typedef float ln4_t __attribute__((ext_vector_type(4)));

// Up to four neighbouring values of a row: element 4 at (VEC: one 16-byte access; else elements at, at + 256, ... one by one), zeros
// past the row's end.
template <bool VEC>
struct LnPlace {
    static __device__ __forceinline__ int element(int group, int i) {
        return VEC ? 4 * ((int)threadIdx.x + LN_THREADS * group) + i : (int)threadIdx.x + LN_THREADS * (4 * group + i);
    }
    static __device__ __forceinline__ ln4_t load(const float* __restrict__ row, int group, int n) {
        if (VEC) {
            const int at = element(group, 0);
            return at < n ? *reinterpret_cast<const ln4_t*>(row + at) : ln4_t{0.0f, 0.0f, 0.0f, 0.0f};
        }
        ln4_t v;
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] = element(group, i) < n ? row[element(group, i)] : 0.0f;
        return v;
    }
    template <typename TO>
    static __device__ __forceinline__ void store(TO* __restrict__ row, int group, int n, const ln4_t& y) {
        if (VEC) {
            const int at = element(group, 0);
            if (at >= n) return;
            if constexpr (sizeof(TO) == 4) *reinterpret_cast<ln4_t*>(row + at) = y;
            else {
                typedef uint32_t u32x2_ln __attribute__((ext_vector_type(2)));
                *reinterpret_cast<u32x2_ln*>(row + at) = u32x2_ln{(uint32_t)f32_to_bf16(y[0]) | ((uint32_t)f32_to_bf16(y[1]) << 16),
                                                                  (uint32_t)f32_to_bf16(y[2]) | ((uint32_t)f32_to_bf16(y[3]) << 16)};
            }
            return;
        }
#pragma unroll
        for (int i = 0; i < 4; ++i)
            if (element(group, i) < n) st(row + element(group, i), y[i]);
    }
};

// mean and 1 / sqrt(var + eps) of a row whose groups get(0), get(1), ... gives
template <bool VEC, typename Get>
__device__ __forceinline__ void row_moments(Get get, int groups, int n, float eps, float* scratch, float& mean, float& rstd) {
    float s = 0.0f;
    for (int j = 0; j < groups; ++j) {
        const ln4_t v = get(j);
        if (VEC) s += (v[0] + v[1]) + (v[2] + v[3]);
        else s = (((s + v[0]) + v[1]) + v[2]) + v[3];
    }
    mean = block_sum<LN_THREADS / 64>(s, scratch) / (float)n;
    float q = 0.0f;
    for (int j = 0; j < groups; ++j) {
        const ln4_t v = get(j);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const float d = LnPlace<VEC>::element(j, i) < n ? v[i] - mean : 0.0f;
            q = fmaf(d, d, q);
        }
    }
    rstd = 1.0f / sqrtf(block_sum<LN_THREADS / 64>(q, scratch) / (float)n + eps);
}

__device__ __forceinline__ ln4_t ln_apply(const ln4_t& v, float mean, float rstd, const ln4_t& w) {
    return ln4_t{(v[0] - mean) * rstd * w[0], (v[1] - mean) * rstd * w[1], (v[2] - mean) * rstd * w[2], (v[3] - mean) * rstd * w[3]};
}

// The row in registers (KEPT groups, with the weights and what else the end needs asked for together at the start), or read again.
// out[r] = LN(x[pick ? pick[r] : r]) in the activation type and/or float32
template <typename TO, int KEPT, bool VEC>
__global__ void __launch_bounds__(LN_THREADS) layernorm_kernel(const float* __restrict__ x, const int* __restrict__ pick, const float* __restrict__ w,
                                                             const float* __restrict__ bias, float eps, TO* __restrict__ out, float* __restrict__ out32, int n) {
    typedef LnPlace<VEC> P;
    __shared__ float scratch[LN_THREADS / 64];
    const int r = blockIdx.x;
    const float* row = x + (size_t)(pick ? pick[r] : r) * n;
    float mean, rstd;
    auto finish = [&](int j, const ln4_t& v, const ln4_t& wj, const ln4_t& bj) {
        ln4_t y = ln_apply(v, mean, rstd, wj);
        if (bias) y = ln4_t{y[0] + bj[0], y[1] + bj[1], y[2] + bj[2], y[3] + bj[3]};
        if (out) P::store(out + (size_t)r * n, j, n, y);
        if (out32) P::store(out32 + (size_t)r * n, j, n, y);
    };
    if (KEPT > 0) {
        ln4_t v[KEPT > 0 ? KEPT : 1], wk[KEPT > 0 ? KEPT : 1], bk[KEPT > 0 ? KEPT : 1];
#pragma unroll
        for (int j = 0; j < KEPT; ++j) {
            v[j] = P::load(row, j, n);
            wk[j] = P::load(w, j, n);
            bk[j] = bias ? P::load(bias, j, n) : ln4_t{0.0f, 0.0f, 0.0f, 0.0f};
        }
        row_moments<VEC>([&](int j) { return v[j]; }, KEPT, n, eps, scratch, mean, rstd);
#pragma unroll
        for (int j = 0; j < KEPT; ++j) finish(j, v[j], wk[j], bk[j]);
    } else {
        const int groups = (n + 4 * LN_THREADS - 1) / (4 * LN_THREADS);
        row_moments<VEC>([&](int j) { return P::load(row, j, n); }, groups, n, eps, scratch, mean, rstd);
        for (int j = 0; j < groups; ++j) finish(j, P::load(row, j, n), P::load(w, j, n), bias ? P::load(bias, j, n) : ln4_t{0.0f, 0.0f, 0.0f, 0.0f});
    }
}

static bool ln_vec(int n, const void* a, const void* b, const void* c, const void* d, const void* e) {
    return n % 4 == 0 && (((uintptr_t)a | (uintptr_t)b | (uintptr_t)c | (uintptr_t)d | (uintptr_t)e) & 15) == 0;
}
// groups of four values a thread keeps: 1, 2 or 4; 0: the row is too long
static int ln_kept(int n) { return n <= 4 * LN_THREADS ? 1 : n <= 8 * LN_THREADS ? 2 : n <= 4 * LN_THREADS * LN_QUADS ? LN_QUADS : 0; }
#define LN_FORMS(TO)                                                            \
    do {                                                                        \
        if (vec) { if (kept == 1) LLMX_LN(TO, 1, true); else if (kept == 2) LLMX_LN(TO, 2, true); else if (kept) LLMX_LN(TO, LN_QUADS, true); else LLMX_LN(TO, 0, true); } \
        else { if (kept == 1) LLMX_LN(TO, 1, false); else if (kept == 2) LLMX_LN(TO, 2, false); else if (kept) LLMX_LN(TO, LN_QUADS, false); else LLMX_LN(TO, 0, false); } \
    } while (0)

extern "C" int llmx_layernorm(const float* x, const int* pick, const float* w, const float* bias, float eps, void* out, int out_dtype, float* out32, int rows, int n,
                              hipStream_t stream) {
    if (rows <= 0) return 0;
    if (n <= 0 || !w || (!out && !out32)) return -2;
    llmx_note_launch(LK_LAYERNORM);
    const int kept = ln_kept(n);
    const bool vec = bias && ln_vec(n, x, w, bias, out, out32);
#define LLMX_LN(TO, K, V) hipLaunchKernelGGL((layernorm_kernel<TO, K, V>), dim3(rows), dim3(LN_THREADS), 0, stream, x, pick, w, bias, eps, (TO*)out, out32, n)
    if (out_dtype == LLMX_F32) LN_FORMS(float);
    else LN_FORMS(bf16_t);
#undef LLMX_LN
    return LLMX_CHECK_LAUNCH();
}

// x[r] += LN(y[r]) * w: a sublayer's result joins the residual after its own norm; `copy` (optional) receives the new row
// in the activation type for the product that reads it next.
template <typename TO, int KEPT, bool VEC>
__global__ void __launch_bounds__(LN_THREADS) layernorm_add_kernel(float* __restrict__ x, const float* __restrict__ y, const float* __restrict__ w,
                                                                 float eps, TO* __restrict__ copy, int n) {
    typedef LnPlace<VEC> P;
    __shared__ float scratch[LN_THREADS / 64];
    const int r = blockIdx.x;
    const float* row = y + (size_t)r * n;
    float* xr = x + (size_t)r * n;
    float mean, rstd;
    auto finish = [&](int j, const ln4_t& v, const ln4_t& wj, const ln4_t& old) {
        const ln4_t z = ln_apply(v, mean, rstd, wj);
        const ln4_t s = ln4_t{old[0] + z[0], old[1] + z[1], old[2] + z[2], old[3] + z[3]};
        P::store(xr, j, n, s);
        if (copy) P::store(copy + (size_t)r * n, j, n, s);
    };
    if (KEPT > 0) {
        ln4_t v[KEPT > 0 ? KEPT : 1], wk[KEPT > 0 ? KEPT : 1], old[KEPT > 0 ? KEPT : 1];
#pragma unroll
        for (int j = 0; j < KEPT; ++j) {
            v[j] = P::load(row, j, n);
            old[j] = P::load(xr, j, n);
            wk[j] = P::load(w, j, n);
        }
        row_moments<VEC>([&](int j) { return v[j]; }, KEPT, n, eps, scratch, mean, rstd);
#pragma unroll
        for (int j = 0; j < KEPT; ++j) finish(j, v[j], wk[j], old[j]);
    } else {
        const int groups = (n + 4 * LN_THREADS - 1) / (4 * LN_THREADS);
        row_moments<VEC>([&](int j) { return P::load(row, j, n); }, groups, n, eps, scratch, mean, rstd);
        for (int j = 0; j < groups; ++j) finish(j, P::load(row, j, n), P::load(w, j, n), P::load(xr, j, n));
    }
}

extern "C" int llmx_layernorm_add(float* x, const float* y, const float* w, float eps, void* copy, int copy_dtype, int rows, int n,
                                  hipStream_t stream) {
    if (rows <= 0) return 0;
    if (n <= 0 || !w) return -2;
    llmx_note_launch(LK_LAYERNORM_ADD);
    const int kept = ln_kept(n);
    const bool vec = false;      // no bias: see above
#define LLMX_LN(TO, K, V) hipLaunchKernelGGL((layernorm_add_kernel<TO, K, V>), dim3(rows), dim3(LN_THREADS), 0, stream, x, y, w, eps, (TO*)copy, n)
    if (copy_dtype == LLMX_F32) LN_FORMS(float);
    else LN_FORMS(bf16_t);
#undef LLMX_LN
    return LLMX_CHECK_LAUNCH();
}

// out = x in the activation type: the rows a product reads when a sublayer takes the residual itself.
template <typename TO>
__global__ void __launch_bounds__(256) cast_rows_kernel(const float* __restrict__ x, TO* __restrict__ out, size_t total) {
    typedef float f32x4_t __attribute__((ext_vector_type(4)));
    const size_t at = 4 * ((size_t)blockIdx.x * 256 + threadIdx.x);
    if (at >= total) return;
    if (at + 4 <= total) {
        const f32x4_t v = *reinterpret_cast<const f32x4_t*>(x + at);
#pragma unroll
        for (int i = 0; i < 4; ++i) st(out + at + i, v[i]);
        return;
    }
    for (size_t i = at; i < total; ++i) st(out + i, x[i]);
}

extern "C" int llmx_cast_rows(const float* x, void* out, int out_dtype, long total, hipStream_t stream) {
    if (total <= 0) return 0;
    llmx_note_launch(LK_CAST_ROWS);
    const dim3 grid((unsigned)((total + 1023) / 1024));
    if (out_dtype == LLMX_F32) hipLaunchKernelGGL(cast_rows_kernel<float>, grid, dim3(256), 0, stream, x, (float*)out, (size_t)total);
    else hipLaunchKernelGGL(cast_rows_kernel<bf16_t>, grid, dim3(256), 0, stream, x, (bf16_t*)out, (size_t)total);
    return LLMX_CHECK_LAUNCH();
}

// out[t] = [x[t] | y[t]] in the activation type, x and y float32 rows of n values: what a product of two joined streams reads.
// y null: only the first half is written (the second is there from before).
template <typename TO, int PER>
__global__ void __launch_bounds__(256) join_rows_kernel(const float* __restrict__ x, const float* __restrict__ y, TO* __restrict__ out, int n, size_t total) {
    const size_t at = PER * ((size_t)blockIdx.x * 256 + threadIdx.x);
    if (at >= total) return;
    const size_t t = at / (size_t)n, i = at % (size_t)n;       // PER divides n: a thread's values lie in one row
    TO* row = out + t * 2 * (size_t)n;
    float a[PER], b[PER];
#pragma unroll
    for (int u = 0; u < PER; ++u) a[u] = x[at + u];
    if (y) {
#pragma unroll
        for (int u = 0; u < PER; ++u) b[u] = y[at + u];
    }
#pragma unroll
    for (int u = 0; u < PER; ++u) st(row + i + u, a[u]);
    if (y) {
#pragma unroll
        for (int u = 0; u < PER; ++u) st(row + n + i + u, b[u]);
    }
}

extern "C" int llmx_join_rows(const float* x, const float* y, void* out, int out_dtype, int rows, int n, hipStream_t stream) {
    if (rows <= 0 || n <= 0) return 0;
    llmx_note_launch(LK_JOIN_ROWS);
    const size_t total = (size_t)rows * n;
    const int per = n % 4 == 0 ? 4 : 1;
    const dim3 grid((unsigned)((total / per + 255) / 256));
    if (out_dtype == LLMX_F32) {
        if (per == 4) hipLaunchKernelGGL((join_rows_kernel<float, 4>), grid, dim3(256), 0, stream, x, y, (float*)out, n, total);
        else hipLaunchKernelGGL((join_rows_kernel<float, 1>), grid, dim3(256), 0, stream, x, y, (float*)out, n, total);
    } else {
        if (per == 4) hipLaunchKernelGGL((join_rows_kernel<bf16_t, 4>), grid, dim3(256), 0, stream, x, y, (bf16_t*)out, n, total);
        else hipLaunchKernelGGL((join_rows_kernel<bf16_t, 1>), grid, dim3(256), 0, stream, x, y, (bf16_t*)out, n, total);
    }
    return LLMX_CHECK_LAUNCH();
}

// out[t, :] = x[t, col0 : col0 + n] in the activation type: some columns of a wider float32 projection as the rows a further
// product reads (the inner values of a low-rank projection).
template <typename TO>
__global__ void __launch_bounds__(256) cast_cols_kernel(const float* __restrict__ x, int ld, TO* __restrict__ out, int n, size_t total) {
    const size_t at = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (at >= total) return;
    st(out + at, x[(at / (size_t)n) * (size_t)ld + (at % (size_t)n)]);
}

extern "C" int llmx_cast_cols(const float* x, int ld, void* out, int out_dtype, int rows, int n, hipStream_t stream) {
    if (rows <= 0 || n <= 0) return 0;
    if (ld < n) return -2;
    llmx_note_launch(LK_CAST_COLS);
    const size_t total = (size_t)rows * n;
    const dim3 grid((unsigned)((total + 255) / 256));
    if (out_dtype == LLMX_F32) hipLaunchKernelGGL(cast_cols_kernel<float>, grid, dim3(256), 0, stream, x, ld, (float*)out, n, total);
    else hipLaunchKernelGGL(cast_cols_kernel<bf16_t>, grid, dim3(256), 0, stream, x, ld, (bf16_t*)out, n, total);
    return LLMX_CHECK_LAUNCH();
}

// out (=, +=) sa * (a + bias_a) + sb * b over float32 rows [T, n]: the join of mixers that run side by side, and a
// projection's bias; bias_a and b may be null.
__global__ void __launch_bounds__(256) combine_rows_kernel(float* __restrict__ out, const float* __restrict__ a, float sa,
                                                         const float* __restrict__ bias_a, const float* __restrict__ b, float sb, int accumulate,
                                                         int n, size_t total) {
    const size_t at = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (at >= total) return;
    float va = a[at];
    if (bias_a) va = va + bias_a[(int)(at % (size_t)n)];
    float v = sa * va;
    if (b) v = v + sb * b[at];
    out[at] = accumulate ? out[at] + v : v;
}

extern "C" int llmx_combine_rows(float* out, const float* a, float sa, const float* bias_a, const float* b, float sb, int accumulate, int rows, int n,
                                 hipStream_t stream) {
    if (rows <= 0 || n <= 0) return 0;
    if (!a) return -2;
    llmx_note_launch(LK_COMBINE_ROWS);
    const size_t total = (size_t)rows * n;
    hipLaunchKernelGGL(combine_rows_kernel, dim3((unsigned)((total + 255) / 256)), dim3(256), 0, stream, out, a, sa, bias_a, b, sb, accumulate, n, total);
    return LLMX_CHECK_LAUNCH();
}

// logits <- logits * scale, then cap * tanh(logits / cap) when cap > 0, in place.
__global__ void __launch_bounds__(256) scale_softcap_kernel(float* __restrict__ z, float scale, float cap, size_t total) {
    const size_t at = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (at >= total) return;
    float v = z[at] * scale;
    if (cap > 0.0f) v = cap * tanhf(v / cap);
    z[at] = v;
}

extern "C" int llmx_scale_softcap(float* z, float scale, float cap, long total, hipStream_t stream) {
    if (total <= 0) return 0;
    llmx_note_launch(LK_SCALE_SOFTCAP);
    hipLaunchKernelGGL(scale_softcap_kernel, dim3((unsigned)((total + 255) / 256)), dim3(256), 0, stream, z, scale, cap, (size_t)total);
    return LLMX_CHECK_LAUNCH();
}
