// Latent attention: the cache keeps, for every token, one latent vector of C values (shared by all heads, RMS-normed)
// followed by one rotated key part of R values.  A head's key for a token is [W_uk_h c | k_rot] and its value W_uv_h c;
// neither is ever formed: the query's unrotated part is taken through W_uk_h^T first (q_lat = W_uk_h^T q_plain, C values),
// so that score = (q_lat . c + q_rot . k_rot) * scale, and the weighted sum of latents goes through W_uv_h afterwards.
// Both products with W_uk / W_uv are grouped products (one group a head) outside this file; here are the step before
// them (norm, rotation, cache write, queries laid out head by head), the attention over the paged latents, and the
// per-head output gate.
//
// Layouts: proj [T, ldp] float32 holds q (H heads of [D unrotated | R rotated]) at column 0 and [C latent | R key part]
// at column q_width; cache [pages, page_tokens, ldc] with the C + R values of a token first in its row (ldc >= C + R; what
// lies behind stays zero); q_plain [H, T, D], q_rot [H, T, R], q_lat and the attention's result [H, T, C] (head-major, so
// that a head's rows are one group of the grouped products), or the same with the first two axes swapped (row-major:
// the grouped products then pick a head's rows by number).  Queries that come through a latent of their own are a product
// of a second matrix with normed rows: the projection then holds [query latent | C | R] and the queries another buffer.
#include "common.h"

struct LatentPrepArgs {
    const float* q;         // [T, ldq]: the heads' queries, at its start
    const float* down;      // [T, ldd]: latent and key part at its start
    const float* q_down;    // [T, ldd] or null: a latent of Cq values that the queries come through
    const float* q_norm_w;  // [Cq]
    void* q_normed;         // [T, Cq]: its norm, in the activation type
    const float* norm_w;    // [C]
    const float* cos_sin;   // [positions, dims]: cos of the dims/2 pairs, then sin (any magnitude factor already inside)
    const int* pos;
    const int* row_entry;
    const int* tables;
    void* q_plain;
    void* q_rot;
    void* cache;
    void* cache_t;          // null, or a second copy of the latents [pages, C, page_tokens] (transposed within the page)
    float eps;
    int T, ldq, ldd, H, D, R, C, Cq, ldc, dims, page_tokens, max_blocks, write_cache;
    int first_role;         // blockIdx.y counts from here: 0 queries, 1 latent and key part, 2 the query latent's norm
    int halves, row_major;
};

// Element r of a rotated part `part` (R values, the first `dims` of them rotated as interleaved pairs (2i, 2i+1) by the
// angle of frequency i): (u, v) -> (u cos - v sin, v cos + u sin).
__device__ __forceinline__ float rotated_interleaved(const float* __restrict__ part, const float* __restrict__ cs, int r, int dims) {
    const float x = part[r];
    if (r >= dims) return x;
    const bool first = (r & 1) == 0;
    const float y = part[first ? r + 1 : r - 1];
    const float c = cs[r >> 1], s = cs[dims / 2 + (r >> 1)];
    return first ? fmaf(-y, s, x * c) : fmaf(y, s, x * c);
}
// The same for pairs (i, i + dims/2).
__device__ __forceinline__ float rotated_part(const float* __restrict__ part, const float* __restrict__ cs, int r, int dims, int halves) {
    if (!halves) return rotated_interleaved(part, cs, r, dims);
    const float x = part[r];
    if (r >= dims) return x;
    const int half = dims / 2;
    const bool first = r < half;
    const int i = first ? r : r - half;
    const float y = part[first ? r + half : i];
    const float c = cs[i], s = cs[half + i];
    return first ? fmaf(-y, s, x * c) : fmaf(y, s, x * c);
}

template <typename TQ, typename TC>
__global__ void __launch_bounds__(256) latent_prep_kernel(LatentPrepArgs a) {
    __shared__ float scratch[4];
    const int t = blockIdx.x, role = a.first_role + blockIdx.y;
    const int p = a.pos[t];
    const float* cs = a.cos_sin + (size_t)p * a.dims;
    const int DR = a.D + a.R;
    if (role == 0) {
        const float* row = a.q + (size_t)t * a.ldq;
        TQ* qp = (TQ*)a.q_plain;
        TQ* qr = (TQ*)a.q_rot;
        int h = threadIdx.x / DR, d = threadIdx.x % DR;
        const int step_h = 256 / DR, step_d = 256 % DR;
        for (int i = threadIdx.x; i < a.H * DR; i += 256) {
            const size_t at = a.row_major ? (size_t)t * a.H + h : (size_t)h * a.T + t;
            if (d < a.D) st(qp + at * a.D + d, row[i]);
            else st(qr + at * a.R + (d - a.D), rotated_part(row + h * DR + a.D, cs, d - a.D, a.dims, a.halves));
            h += step_h;
            d += step_d;
            if (d >= DR) {
                d -= DR;
                ++h;
            }
        }
        return;
    }
    if (role == 2) {
        const float* lat = a.q_down + (size_t)t * a.ldd;
        const float s = block_sum<4>(strided_squares<256>(lat, a.Cq), scratch);
        const float r = 1.0f / sqrtf(s / (float)a.Cq + a.eps);
        TQ* out = (TQ*)a.q_normed + (size_t)t * a.Cq;
        for (int i = threadIdx.x; i < a.Cq; i += 256) st(out + i, lat[i] * (r * a.q_norm_w[i]));
        return;
    }
    if (!a.write_cache) return;
    const float* lat = a.down + (size_t)t * a.ldd;
    const float s = block_sum<4>(strided_squares<256>(lat, a.C), scratch);
    const float r = 1.0f / sqrtf(s / (float)a.C + a.eps);
    const int page = a.tables[(size_t)a.row_entry[t] * a.max_blocks + p / a.page_tokens];
    TC* out = (TC*)a.cache + ((size_t)page * a.page_tokens + p % a.page_tokens) * a.ldc;
    TC* out_t = a.cache_t ? (TC*)a.cache_t + (size_t)page * a.C * a.page_tokens + p % a.page_tokens : nullptr;
    for (int i = threadIdx.x; i < a.C; i += 256) {
        const float c = lat[i] * (r * a.norm_w[i]);
        st(out + i, c);
        if (out_t) st(out_t + (size_t)i * a.page_tokens, c);
    }
    for (int i = threadIdx.x; i < a.R; i += 256) st(out + a.C + i, rotated_part(lat + a.C, cs, i, a.dims, a.halves));
}

static int launch_latent_prep(const LatentPrepArgs& a, int roles, int dtype, hipStream_t stream) {
    llmx_note_launch(LK_LATENT_PREP);
    if (dtype == LLMX_F32) hipLaunchKernelGGL((latent_prep_kernel<float, float>), dim3(a.T, roles), dim3(256), 0, stream, a);
    else hipLaunchKernelGGL((latent_prep_kernel<bf16_t, bf16_t>), dim3(a.T, roles), dim3(256), 0, stream, a);
    return LLMX_CHECK_LAUNCH();
}

extern "C" int llmx_latent_prep(const float* proj, const float* norm_w, const float* cos_sin, const int* pos, const int* row_entry,
                                const int* tables, void* q_plain, void* q_rot, void* cache, void* cache_t, int dtype, float eps, int T, int ldp, int H, int D,
                                int R, int C, int ldc, int dims, int page_tokens, int max_blocks, int write_cache, int halves, int row_major,
                                hipStream_t stream) {
    if (T <= 0) return 0;
    if (dims % 2 || dims > R || D + R <= 0 || C <= 0 || H * (D + R) + C + R > ldp || ldc < C + R) return -2;
    LatentPrepArgs a{proj, proj + H * (D + R), nullptr, nullptr, nullptr, norm_w, cos_sin, pos, row_entry, tables, q_plain, q_rot, cache, cache_t,
                     eps, T, ldp, ldp, H, D, R, C, 0, ldc, dims, page_tokens, max_blocks, write_cache, 0, halves, row_major};
    return launch_latent_prep(a, 2, dtype, stream);
}

// The same in two steps for queries that come through a latent of their own: proj [T, ldp] = [Cq query latent | C | R].  First
// the norms: the query latent's into q_normed (what the second query product reads), the cached latent with its key part
// into the row's page; then, after that product, its rows q [T, H (D + R)] laid out and rotated.
extern "C" int llmx_latent_down(const float* proj, const float* q_norm_w, void* q_normed, const float* norm_w, const float* cos_sin, const int* pos,
                                const int* row_entry, const int* tables, void* cache, void* cache_t, int dtype, float eps, int T, int ldp, int Cq,
                                int R, int C, int ldc, int dims, int page_tokens, int max_blocks, int write_cache, int halves, hipStream_t stream) {
    if (T <= 0) return 0;
    if (dims % 2 || dims > R || C <= 0 || Cq <= 0 || Cq + C + R > ldp || ldc < C + R) return -2;
    LatentPrepArgs a{nullptr, proj + Cq, proj, q_norm_w, q_normed, norm_w, cos_sin, pos, row_entry, tables, nullptr, nullptr, cache, cache_t,
                     eps, T, 0, ldp, 1, 1, R, C, Cq, ldc, dims, page_tokens, max_blocks, write_cache, 1, halves, 0};
    return launch_latent_prep(a, 2, dtype, stream);
}

extern "C" int llmx_latent_queries(const float* q, const float* cos_sin, const int* pos, void* q_plain, void* q_rot, int dtype, int T, int ldq, int H,
                                   int D, int R, int dims, int halves, int row_major, hipStream_t stream) {
    if (T <= 0) return 0;
    if (dims % 2 || dims > R || D + R <= 0 || H * (D + R) > ldq) return -2;
    LatentPrepArgs a{q, nullptr, nullptr, nullptr, nullptr, nullptr, cos_sin, pos, nullptr, nullptr, q_plain, q_rot, nullptr, nullptr,
                     0.0f, T, ldq, 0, H, D, R, 1, 0, 1, dims, 1, 1, 0, 0, halves, row_major};
    return launch_latent_prep(a, 1, dtype, stream);
}

// ---------------------------------------------------------------------------
// The universal kernel: one wave per (row, head).  Keys lo..p of the row's request are walked in tiles of 64 absolute
// positions with an online softmax; lane j of a tile forms the score of key 64*tile + j, for the weighted sum lane d
// owns latent dims d, d + 64, ... and walks the tile's keys in order.  A row's arithmetic depends on its own position
// and request only.  Any sizes with C <= 2048 and C + R <= 4096, float32 or bfloat16.
struct LatentAttnArgs {
    const void* q_lat;   // [H, T, C]
    const void* q_rot;   // [H, T, R]
    const void* cache;   // [pages, page_tokens, ldc]
    const int* pos;
    const int* row_entry;
    const int* tables;
    void* out;           // [H, T, C]
    float scale;
    int T, H, C, R, ldc, page_tokens, max_blocks, window, row_major;
    const float* sink;   // [H] or null: one more logit a head in the denominator, with no key and no value
};

#define LAT_MAX_C 2048
#define LAT_MAX_CR 4096

template <typename T>
__global__ void __launch_bounds__(64) latent_attention_generic_kernel(LatentAttnArgs a) {
    __shared__ float qs[LAT_MAX_CR];
    __shared__ float ps[64];
    __shared__ int row_at[64];   // page * page_tokens + slot of each key of the tile
    const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
    const int C = a.C, R = a.R, CR = C + R;
    const int p = a.pos[t];
    const int* table = a.tables + (size_t)a.row_entry[t] * a.max_blocks;
    const size_t q_at = a.row_major ? (size_t)t * a.H + h : (size_t)h * a.T + t;
    const T* ql = (const T*)a.q_lat + q_at * C;
    const T* qr = (const T*)a.q_rot + q_at * R;
    const T* cache = (const T*)a.cache;
    for (int d = lane; d < C; d += 64) qs[d] = ld(ql + d);
    for (int d = lane; d < R; d += 64) qs[C + d] = ld(qr + d);
    __syncthreads();

    int lo = (a.window > 0 && p - a.window + 1 > 0) ? p - a.window + 1 : 0;
    float m = -INFINITY, l = 0.0f;
    float acc[LAT_MAX_C / 64];
#pragma unroll
    for (int i = 0; i < LAT_MAX_C / 64; ++i) acc[i] = 0.0f;

    for (int j0 = (lo / 64) * 64; j0 <= p; j0 += 64) {
        const int j = j0 + lane;
        const bool seen = j >= lo && j <= p;
        float s = -INFINITY;
        int at = 0;
        if (seen) {
            at = table[j / a.page_tokens] * a.page_tokens + j % a.page_tokens;
            const T* key = cache + (size_t)at * a.ldc;
            float dot = 0.0f;
            for (int d = 0; d < CR; ++d) dot = fmaf(qs[d], ld(key + d), dot);
            s = dot * a.scale;
        }
        const float m_new = fmaxf(m, wave_max(s));
        const float w = seen ? expf(s - m_new) : 0.0f;
        const float correction = expf(m - m_new);   // 0 on the first tile (m = -inf)
        ps[lane] = w;
        row_at[lane] = at;
        __syncthreads();
        const int n = min(64, p - j0 + 1);
        float tile_sum = 0.0f;
        for (int i = 0; i < n; ++i) tile_sum += ps[i];   // keys before lo hold 0
        l = l * correction + tile_sum;
#pragma unroll
        for (int i = 0; i < LAT_MAX_C / 64; ++i) {
            const int d = lane + 64 * i;
            if (d < C) {
                float v = acc[i] * correction;
                for (int jj = 0; jj < n; ++jj) v = fmaf(ps[jj], ld(cache + (size_t)row_at[jj] * a.ldc + d), v);
                acc[i] = v;
            }
        }
        m = m_new;
        __syncthreads();
    }
    float shrink = 1.0f;
    if (a.sink) {
        const float top = fmaxf(m, a.sink[h]);
        shrink = expf(m - top);
        l = l * shrink + expf(a.sink[h] - top);
    }
    T* out = (T*)a.out + q_at * C;
#pragma unroll
    for (int i = 0; i < LAT_MAX_C / 64; ++i) {
        const int d = lane + 64 * i;
        if (d < C) st(out + d, a.sink ? acc[i] * shrink / l : acc[i] / l);
    }
}

extern "C" int llmx_latent_attention_generic(const void* q_lat, const void* q_rot, const void* cache, const int* pos, const int* row_entry,
                                             const int* tables, void* out, int dtype, float scale, int T, int H, int C, int R, int ldc, int page_tokens,
                                             int max_blocks, int window, int row_major, const float* sink, hipStream_t stream) {
    if (T <= 0 || H <= 0) return 0;
    if (C <= 0 || C > LAT_MAX_C || R < 0 || C + R > LAT_MAX_CR || ldc < C + R) return -2;
    llmx_note_launch(LK_LATENT_ATTENTION_GENERIC);
    LatentAttnArgs a{q_lat, q_rot, cache, pos, row_entry, tables, out, scale, T, H, C, R, ldc, page_tokens, max_blocks, window, row_major, sink};
    if (dtype == LLMX_F32) hipLaunchKernelGGL(latent_attention_generic_kernel<float>, dim3(T, H), dim3(64), 0, stream, a);
    else hipLaunchKernelGGL(latent_attention_generic_kernel<bf16_t>, dim3(T, H), dim3(64), 0, stream, a);
    return LLMX_CHECK_LAUNCH();
}

// ---------------------------------------------------------------------------
// Per-head output gate and the change of layout before the output projection:
// out[t, h*V + d] = sigmoid(gate[t*ldg + h]) * values[h, t, d], values float32 [H, T, V], out in the activation type.
template <typename TO>
__global__ void __launch_bounds__(256) head_gate_kernel(const float* __restrict__ values, const float* __restrict__ gate, int ldg,
                                                      TO* __restrict__ out, int T, int H, int V) {
    const int t = blockIdx.x;
    int h = threadIdx.x / V, d = threadIdx.x % V;
    const int step_h = 256 / V, step_d = 256 % V;
    for (int i = threadIdx.x; i < H * V; i += 256) {
        const float g = gate ? 1.0f / (1.0f + expf(-gate[(size_t)t * ldg + h])) : 1.0f;
        st(out + (size_t)t * H * V + i, g * values[((size_t)h * T + t) * V + d]);
        h += step_h;
        d += step_d;
        if (d >= V) {
            d -= V;
            ++h;
        }
    }
}

extern "C" int llmx_head_gate(const float* values, const float* gate, int ldg, void* out, int out_dtype, int T, int H, int V, hipStream_t stream) {
    if (T <= 0 || H <= 0 || V <= 0) return 0;
    llmx_note_launch(LK_HEAD_GATE);
    if (out_dtype == LLMX_F32) hipLaunchKernelGGL(head_gate_kernel<float>, dim3(T), dim3(256), 0, stream, values, gate, ldg, (float*)out, T, H, V);
    else hipLaunchKernelGGL(head_gate_kernel<bf16_t>, dim3(T), dim3(256), 0, stream, values, gate, ldg, (bf16_t*)out, T, H, V);
    return LLMX_CHECK_LAUNCH();
}
