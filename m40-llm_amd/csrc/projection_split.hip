// Steps between a mixer's projections and what it does with them.
//
// qkv_split_kernel     attention of one map a head: biases, RMS norm over whole projections, rotation, values mixed with another layer's;
//                      queries out, keys and values to the cache.  A workgroup a row, or several for few rows (each forms the norms).
// delta_split_kernel   delta rule: short convolution and silu, queries and keys as unit vectors; f32 rows out.  A workgroup takes 16 rows of
//                      one head.
#include "packed_gemm.hpp"
#include "pair_cache.hpp"
#include "short_conv.hpp"

namespace {

constexpr uint32_t kThreads = 256;

__device__ __forceinline__ float2 block_sum2(float2 v, float2* scratch) {
    v.x = m40_sum64(v.x);
    v.y = m40_sum64(v.y);
    if ((threadIdx.x & 63u) == 0u) scratch[threadIdx.x >> 6] = v;
    __syncthreads();
    float2 s = scratch[0];
#pragma unroll
    for (uint32_t i = 1; i < kThreads / 64; ++i) {
        s.x += scratch[i].x;
        s.y += scratch[i].y;
    }
    return s;
}

// Four neighbouring columns a thread at a time (W 4), or one.
template <class T, int W>
__global__ __launch_bounds__(kThreads) void qkv_split_kernel(M40llmQkvSplit a, M40PairPage page) {
    __shared__ float2 scratch[kThreads / 64];
    const uint32_t row = m40_tile_row(blockIdx.x, a.rows), tid = threadIdx.x;
    const float* proj = static_cast<const float*>(a.proj) + (size_t)row * a.ld_proj;
    const uint32_t pos = a.row_pos[row];
    const uint32_t number = a.page_table[(size_t)a.row_slot[row] * a.max_pages + pos / M40LLM_PAGE_TOKENS], t = pos % M40LLM_PAGE_TOKENS;
    auto biased = [&](uint32_t offset, const void* bias, uint32_t c) __attribute__((always_inline)) {
        M40Columns<W> v = m40_load_columns<W>(proj + offset + c);
        if (bias) {
            const M40Columns<W> b = m40_load_columns<W>(static_cast<const float*>(bias) + c);
#pragma unroll
            for (int k = 0; k < W; ++k) v.v[k] += b.v[k];
        }
        return v;
    };
    const uint32_t q_cols = a.heads * a.dim, k_cols = a.kv_heads * a.dim;
    float q_inv = 1.0f, k_inv = 1.0f;
    if (a.q_norm) {
        float2 ss = {0.0f, 0.0f};
        for (uint32_t c = tid * W; c < q_cols; c += kThreads * W) {
            const M40Columns<W> v = biased(0u, a.q_bias, c);
#pragma unroll
            for (int k = 0; k < W; ++k) ss.x = fmaf(v.v[k], v.v[k], ss.x);
        }
        for (uint32_t c = tid * W; c < k_cols; c += kThreads * W) {
            const M40Columns<W> v = biased(a.k_offset, a.k_bias, c);
#pragma unroll
            for (int k = 0; k < W; ++k) ss.y = fmaf(v.v[k], v.v[k], ss.y);
        }
        ss = block_sum2(ss, scratch);
        q_inv = 1.0f / sqrtf(ss.x / (float)q_cols + a.eps);
        k_inv = 1.0f / sqrtf(ss.y / (float)k_cols + a.eps);
    }
    const float2* angles = static_cast<const float2*>(a.angles) + (a.angles ? (size_t)row * a.rot_half : 0);
    // columns at .. of head `unit`, normed and rotated; zero past the head
    auto turned = [&](uint32_t offset, const void* bias, const void* norm, float inv, uint32_t unit, uint32_t at, float (&y)[W]) __attribute__((always_inline)) {
#pragma unroll
        for (int k = 0; k < W; ++k) y[k] = 0.0f;
        if (at >= a.dim) return;
        auto normed = [&](uint32_t c) __attribute__((always_inline)) {
            M40Columns<W> v = biased(offset, bias, c);
            if (norm) {
                const M40Columns<W> w = m40_load_columns<W>(static_cast<const float*>(norm) + c);
#pragma unroll
                for (int k = 0; k < W; ++k) v.v[k] *= inv * w.v[k];
            }
            return v;
        };
        const M40Columns<W> v = normed(unit * a.dim + at);
#pragma unroll
        for (int k = 0; k < W; ++k) y[k] = v.v[k];
        if (!angles || at / 2u >= a.rot_half) return;
        if (W == 4) {
#pragma unroll
            for (int k = 0; k < W; k += 2) {
                const float2 cs = (at + k) / 2u < a.rot_half ? angles[(at + k) / 2u] : make_float2(1.0f, 0.0f);
                const float u = v.v[k], w = v.v[W > 1 ? k + 1 : 0];
                y[k] = fmaf(u, cs.x, -(w * cs.y));
                y[W > 1 ? k + 1 : 0] = fmaf(w, cs.x, u * cs.y);
            }
        } else {
            const uint32_t other = at ^ 1u;
            if (other >= a.dim) return;
            const float2 cs = angles[at / 2u];
            const float w = normed(unit * a.dim + other).v[0];
            y[0] = at & 1u ? fmaf(v.v[0], cs.x, w * cs.y) : fmaf(v.v[0], cs.x, -(w * cs.y));
        }
    };
    const uint32_t k_pad = page.k_tiles * 32u, v_pad = page.v_tiles * 16u, first = (blockIdx.y * kThreads + tid) * W;
    T* q = static_cast<T*>(a.queries) + (size_t)row * a.heads * k_pad;
    for (uint32_t i = first; i < a.heads * k_pad; i += kThreads * W * gridDim.y) {
        float y[W];
        turned(0u, a.q_bias, a.q_norm, q_inv * a.q_factor, i / k_pad, i % k_pad, y);
        if (!a.q_norm) {
#pragma unroll
            for (int k = 0; k < W; ++k) y[k] *= a.q_factor;
        }
        m40_store_columns<T, W>(q + i, y);
    }
    T* cache = static_cast<T*>(a.cache) + number * page.elements();
    for (uint32_t i = first; i < a.kv_heads * k_pad; i += kThreads * W * gridDim.y) {
        float y[W];
        turned(a.k_offset, a.k_bias, a.k_norm, k_inv, i / k_pad, i % k_pad, y);
        m40_store_columns<T, W>(cache + i / k_pad * page.head_elements() + page.key_at(0u, t, i % k_pad), y);
    }
    const float lambda = a.lambda;
    for (uint32_t i = first; i < a.kv_heads * v_pad; i += kThreads * W * gridDim.y) {
        const uint32_t unit = i / v_pad, at = i % v_pad, c = unit * a.vdim + at;
        T* to = cache + unit * page.head_elements();
        M40Columns<W> v{};
        if (at < a.vdim) {
            v = biased(a.v_offset, a.v_bias, c);
            if (a.keep_values) m40_store_columns<float, W>(static_cast<float*>(a.keep_values) + (size_t)row * a.ld_values + c, v.v);
            if (a.first_values) {
                const M40Columns<W> f = m40_load_columns<W>(static_cast<const float*>(a.first_values) + (size_t)row * a.ld_values + c);
#pragma unroll
                for (int k = 0; k < W; ++k) v.v[k] = fmaf(lambda, f.v[k], (1.0f - lambda) * v.v[k]);
            }
        }
#pragma unroll
        for (int k = 0; k < W; ++k) to[page.value_at(t, at + k)] = M40Act<T>::from(v.v[k]);
    }
}

// N groups of columns at most a lane
template <int W, int N>
__global__ __launch_bounds__(kThreads) void delta_split_kernel(M40llmDeltaSplit a) {
    const uint32_t row = blockIdx.x * 16u + (threadIdx.x >> 4), lane = threadIdx.x & 15u;
    if (row >= a.rows) return;               // no barrier below; the 16 lanes of a row stay together
    uint32_t unit = blockIdx.y, col0 = 0, n = a.dim, all = a.kv_heads * a.dim;
    const void* conv = a.q_conv;
    float factor = a.q_factor;
    const bool value = unit >= 2u * a.kv_heads;
    if (value) {
        unit -= 2u * a.kv_heads;
        col0 = 2u * a.kv_heads * a.dim; n = a.vdim; all = a.heads * a.vdim; conv = a.v_conv;
    } else if (unit >= a.kv_heads) {
        unit -= a.kv_heads;
        col0 = a.kv_heads * a.dim; conv = a.k_conv; factor = 1.0f;
    }
    col0 += unit * n;
    const uint32_t keep = a.taps - 1u, slot = a.row_slot[row];
    const M40ConvRow r{static_cast<const float*>(a.proj) + (size_t)row * a.ld_proj + col0, (size_t)a.ld_proj, static_cast<const float*>(conv) + unit * n, all, a.taps,
                       keep ? static_cast<float*>(a.conv_state) + (size_t)slot * keep * a.ld_state + col0 : nullptr, (size_t)a.ld_state, a.row_pos[row], a.row_back[row]};
    float y[N][W];
    m40_short_conv<W, N>(r, n, lane, y);
#pragma unroll
    for (int i = 0; i < N; ++i)
#pragma unroll
        for (int k = 0; k < W; ++k) y[i][k] = m40_silu(y[i][k]);
    if (!value) {
        const float f = factor / sqrtf(m40_sum_squares16<W, N>(y) + 1e-6f);
#pragma unroll
        for (int i = 0; i < N; ++i)
#pragma unroll
            for (int k = 0; k < W; ++k) y[i][k] *= f;
    }
    float* out = static_cast<float*>(a.out) + (size_t)row * a.ld_out + col0;
#pragma unroll
    for (int i = 0; i < N; ++i) {
        const uint32_t at = W * (lane + 16u * i);
        if (at < n) m40_store_columns<float, W>(out + at, y[i]);
    }
}

int launched() { return hipGetLastError() == hipSuccess ? 0 : -2; }

}  // namespace

extern "C" {

int m40llm_ext_qkv_split_append_async(M40llmCudaContext* ctx, const M40llmQkvSplit* s, uint32_t stream_kind) {
    if (!ctx || !s || !s->proj || !s->queries || !s->cache || !s->row_slot || !s->row_pos || !s->page_table) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    if (s->rows == 0 || s->act_dtype > 1u || s->heads == 0 || s->kv_heads == 0 || s->heads % s->kv_heads != 0 || s->dim == 0 || s->dim > M40LLM_PAIR_MOST_DIM ||
        s->vdim == 0 || s->vdim > M40LLM_PAIR_MOST_DIM || s->k_offset < s->heads * s->dim || s->v_offset < s->k_offset + s->kv_heads * s->dim ||
        s->ld_proj < (uint64_t)s->v_offset + s->kv_heads * s->vdim || !m40_aligned16(s->queries) || !m40_aligned16(s->cache))
        return -3;
    if ((s->q_norm == nullptr) != (s->k_norm == nullptr) || (s->angles && s->rot_half * 2u > s->dim + 1u) ||
        ((s->first_values || s->keep_values) && s->ld_values < (uint64_t)s->kv_heads * s->vdim))
        return -4;
    const M40PairPage page(1u, s->kv_heads, s->dim, s->vdim);
    bool vec = s->dim % 4u == 0 && s->vdim % 4u == 0 && s->ld_proj % 4u == 0 && s->k_offset % 4u == 0 && s->v_offset % 4u == 0 && s->ld_values % 4u == 0;
    for (const void* p : {s->proj, s->q_bias, s->k_bias, s->v_bias, s->q_norm, s->k_norm, s->first_values, static_cast<const void*>(s->keep_values)})
        vec = vec && m40_aligned16(p);
    // parts of a row's queries
    const uint32_t most = (s->heads * page.k_tiles * 32u + 1023u) / 1024u, parts = s->rows > 64u ? 1u : most < 8u ? most : 8u;
    const dim3 grid(s->rows, parts);
    (void)hipGetLastError();
    if (s->act_dtype == M40LLM_ACT_F32) {
        if (vec) qkv_split_kernel<float, 4><<<grid, kThreads, 0, stream>>>(*s, page);
        else qkv_split_kernel<float, 1><<<grid, kThreads, 0, stream>>>(*s, page);
    } else {
        if (vec) qkv_split_kernel<m40_bf16, 4><<<grid, kThreads, 0, stream>>>(*s, page);
        else qkv_split_kernel<m40_bf16, 1><<<grid, kThreads, 0, stream>>>(*s, page);
    }
    return launched();
}

int m40llm_ext_delta_split_async(M40llmCudaContext* ctx, const M40llmDeltaSplit* s, uint32_t stream_kind) {
    if (!ctx || !s || !s->proj || !s->q_conv || !s->k_conv || !s->v_conv || !s->out || !s->row_slot || !s->row_pos || !s->row_back) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    const uint64_t cols = 2ull * s->kv_heads * s->dim + (uint64_t)s->heads * s->vdim;
    const uint32_t most = s->dim > s->vdim ? s->dim : s->vdim;
    if (s->rows == 0 || s->heads == 0 || s->kv_heads == 0 || s->heads % s->kv_heads != 0 || s->dim == 0 || s->vdim == 0 || most > 256u || s->taps == 0 ||
        2u * s->kv_heads + s->heads > 65535u || s->ld_proj < cols || s->ld_out < cols)
        return -3;
    if (s->taps > 1u && (!s->conv_state || s->ld_state < cols)) return -4;
    bool vec = s->dim % 4u == 0 && s->vdim % 4u == 0 && s->ld_proj % 4u == 0 && s->ld_state % 4u == 0 && s->ld_out % 4u == 0;
    for (const void* p : {s->proj, s->q_conv, s->k_conv, s->v_conv, static_cast<const void*>(s->conv_state), static_cast<const void*>(s->out)}) vec = vec && m40_aligned16(p);
    const dim3 grid((s->rows + 15u) / 16u, 2u * s->kv_heads + s->heads);
    (void)hipGetLastError();
    if (!vec) delta_split_kernel<1, 16><<<grid, kThreads, 0, stream>>>(*s);
    else if (most <= 64u) delta_split_kernel<4, 1><<<grid, kThreads, 0, stream>>>(*s);
    else if (most <= 128u) delta_split_kernel<4, 2><<<grid, kThreads, 0, stream>>>(*s);
    else delta_split_kernel<4, 4><<<grid, kThreads, 0, stream>>>(*s);
    return launched();
}

}  // extern "C"
