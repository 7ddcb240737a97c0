// Row-wise steps of layers whose sublayers have their norm on the output: norm + residual add, norm + gate, and the step between an
// attention's projections and its attention (short convolution, query and key norms, cache append).
#include "packed_gemm.hpp"
#include "pair_cache.hpp"
#include "short_conv.hpp"

namespace {

constexpr int kThreads = 256;

__device__ __forceinline__ float block_sum(float v, float* scratch) {
    v = m40_sum64(v);
    __syncthreads();
    if ((threadIdx.x & 63u) == 0u) scratch[threadIdx.x >> 6] = v;
    __syncthreads();
    float s = scratch[0];
#pragma unroll
    for (int i = 1; i < kThreads / 64; ++i) s += scratch[i];
    return s;
}
template <class T, bool VEC>
__device__ __forceinline__ void load_group(const T* src, uint32_t at, uint32_t width, float (&v)[8]) {
    if (VEC) {
        const typename M40Act<T>::vec8 t = M40Act<T>::load8(src + at);
#pragma unroll
        for (int i = 0; i < 8; ++i) v[i] = M40Act<T>::to(t[i]);
    } else {
#pragma unroll
        for (uint32_t i = 0; i < 8; ++i) v[i] = at + i < width ? M40Act<T>::to(src[at + i]) : 0.0f;
    }
}

// A thread takes groups of eight neighbouring elements and keeps two of them in registers (width up to 4096); beyond, sums are formed again.
template <class T, bool VEC>
__global__ __launch_bounds__(kThreads) void norm_add_rows_kernel(M40llmNormAdd a) {
    __shared__ float scratch[kThreads / 64];
    constexpr uint32_t kGroups = 2;
    const uint32_t row = m40_tile_row(blockIdx.x, a.rows), width = a.width, groups = a.ld_h / 8u;
    float* x = static_cast<float*>(a.x) + (size_t)row * width;
    const float* w = static_cast<const float*>(a.w);
    auto value = [&](uint32_t g, float (&y)[8]) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < 8; ++i) y[i] = 0.0f;
        if (g * 8u >= width) return;
        if (a.place) {
            for (uint32_t j = 0; j < a.top; ++j) {
                const uint32_t at = a.place[(size_t)row * a.top + j];
                const float f = static_cast<const float*>(a.weight)[(size_t)row * a.top + j];
                float v[8];
                if (at == M40LLM_PLACE_INPUT) load_group<float, VEC>(x, g * 8u, width, v);
                else load_group<T, VEC>(static_cast<const T*>(a.expert_out) + (size_t)at * a.ld_expert, g * 8u, width, v);
#pragma unroll
                for (int i = 0; i < 8; ++i) y[i] = fmaf(f, v[i], y[i]);
            }
        } else {
            for (uint32_t p = 0; p < a.n_planes; ++p) {
                float v[8];
                load_group<float, VEC>(static_cast<const float*>(a.planes) + p * (size_t)a.plane_stride + (size_t)row * width, g * 8u, width, v);
#pragma unroll
                for (int i = 0; i < 8; ++i) y[i] += v[i];
            }
        }
    };
    float keep[kGroups][8];
    float q = 0.0f;
    auto sq8 = [&](const float (&y)[8]) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < 8; ++i) q = fmaf(y[i], y[i], q);
    };
#pragma unroll
    for (uint32_t j = 0; j < kGroups; ++j) {
        value(threadIdx.x + j * kThreads, keep[j]);
        sq8(keep[j]);
    }
    for (uint32_t g = threadIdx.x + kGroups * kThreads; g < groups; g += kThreads) {
        float y[8];
        value(g, y);
        sq8(y);
    }
    const float f = a.mult / sqrtf(block_sum(q, scratch) / (float)width + a.eps);
    auto finish = [&](uint32_t g, const float (&y)[8]) __attribute__((always_inline)) {
        float v[8];
        if (g * 8u < width) {
            load_group<float, VEC>(x, g * 8u, width, v);
#pragma unroll
            for (uint32_t i = 0; i < 8; ++i) v[i] = VEC || g * 8u + i < width ? fmaf(y[i] * f, w[g * 8u + i], v[i]) : 0.0f;
            if (VEC) {
                reinterpret_cast<float4*>(x + g * 8u)[0] = make_float4(v[0], v[1], v[2], v[3]);
                reinterpret_cast<float4*>(x + g * 8u)[1] = make_float4(v[4], v[5], v[6], v[7]);
            } else {
#pragma unroll
                for (uint32_t i = 0; i < 8; ++i)
                    if (g * 8u + i < width) x[g * 8u + i] = v[i];
            }
        } else {
#pragma unroll
            for (int i = 0; i < 8; ++i) v[i] = 0.0f;
        }
        const m40_float4 lo = {v[0], v[1], v[2], v[3]}, hi = {v[4], v[5], v[6], v[7]};
        T* o = static_cast<T*>(a.h) + m40_packed_at(row, g * 8u, a.ld_h >> 5);
        m40_store4<T>(o, lo);
        m40_store4<T>(o + 4, hi);
        if (a.h_rows) {
            T* r = static_cast<T*>(a.h_rows) + (size_t)row * a.ld_h + g * 8u;
            m40_store4<T>(r, lo);
            m40_store4<T>(r + 4, hi);
        }
    };
#pragma unroll
    for (uint32_t j = 0; j < kGroups; ++j) {
        const uint32_t g = threadIdx.x + j * kThreads;
        if (g < groups) finish(g, keep[j]);
    }
    for (uint32_t g = threadIdx.x + kGroups * kThreads; g < groups; g += kThreads) {
        float y[8];
        value(g, y);
        finish(g, y);
    }
}

template <class T, bool VEC>
__global__ __launch_bounds__(kThreads) void norm_gate_rows_kernel(const float* __restrict__ y, size_t ld_y, const float* __restrict__ w,
                                                                  const float* __restrict__ gate, size_t ld_gate, uint32_t rows, uint32_t cols, float eps,
                                                                  T* __restrict__ out, uint32_t ld_out) {
    __shared__ float scratch[kThreads / 64];
    const uint32_t row = m40_tile_row(blockIdx.x, rows);
    const float *src = y + (size_t)row * ld_y, *gt = gate + (size_t)row * ld_gate;
    float q = 0.0f;
    for (uint32_t g = threadIdx.x; g * 8u < cols; g += kThreads) {
        float v[8];
        load_group<float, VEC>(src, g * 8u, cols, v);
#pragma unroll
        for (int i = 0; i < 8; ++i) q = fmaf(v[i], v[i], q);
    }
    const float inv = 1.0f / sqrtf(block_sum(q, scratch) / (float)cols + eps);
    for (uint32_t g = threadIdx.x; g < ld_out / 8u; g += kThreads) {
        float v[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) v[i] = 0.0f;
        if (g * 8u < cols) {
            float z[8];
            load_group<float, VEC>(src, g * 8u, cols, v);
            load_group<float, VEC>(gt, g * 8u, cols, z);
#pragma unroll
            for (uint32_t i = 0; i < 8; ++i) v[i] = VEC || g * 8u + i < cols ? v[i] * inv * w[g * 8u + i] * m40_sigmoid(z[i]) : 0.0f;
        }
        T* o = out + m40_packed_at(row, g * 8u, ld_out >> 5);
        m40_store4<T>(o, m40_float4{v[0], v[1], v[2], v[3]});
        m40_store4<T>(o + 4, m40_float4{v[4], v[5], v[6], v[7]});
    }
}

// A workgroup takes 16 rows and one unit: a map (of one or two) of a query head, a map of a key head, or a value head; 16 lanes a row.
enum { kQueries = 0, kKeys = 1, kValues = 2 };
template <class T, int W, int N>
__device__ __forceinline__ void split_unit(const M40llmPairSplit& a, const M40PairPage& page, int kind, uint32_t unit, uint32_t row, uint32_t lane) {
    const uint32_t n = kind == kValues ? a.vdim : a.dim, col0 = (kind == kQueries ? 0u : kind == kKeys ? a.k_offset : a.v_offset) + unit * n;
    const uint32_t all = (kind == kQueries ? a.maps * a.heads : kind == kKeys ? a.maps * a.kv_heads : a.kv_heads) * n;      // columns of this kind
    const float* conv = static_cast<const float*>(kind == kQueries ? a.q_conv : kind == kKeys ? a.k_conv : a.v_conv);
    const uint32_t pos = a.row_pos[row], slot = a.row_slot[row], info = a.row_back[row];
    const uint32_t number = kind == kQueries ? 0u : a.page_table[(size_t)slot * a.max_pages + pos / M40LLM_PAGE_TOKENS];
    const uint32_t keep = a.taps ? a.taps - 1u : 0u;
    const M40ConvRow r{static_cast<const float*>(a.proj) + (size_t)row * a.ld_proj + col0, (size_t)a.ld_proj, a.taps ? conv + unit * n : nullptr, all, a.taps,
                       keep ? static_cast<float*>(a.conv_state) + (size_t)slot * keep * a.ld_state + col0 : nullptr, (size_t)a.ld_state, pos, info};
    float y[N][W];
    m40_short_conv<W, N>(r, n, lane, y);
    if (kind != kValues) {
        const float* norm = static_cast<const float*>(kind == kQueries ? a.q_norm : a.k_norm);
        const float inv = 1.0f / sqrtf(m40_sum_squares16<W, N>(y) / (float)n + a.eps);
#pragma unroll
        for (int i = 0; i < N; ++i) {
            const uint32_t c = W * (lane + 16u * i);
            const M40Columns<W> w = m40_load_columns<W>(norm + (c < n ? c : 0u));
#pragma unroll
            for (int k = 0; k < W; ++k) y[i][k] *= inv * w.v[k];
        }
    }
    T* cache = static_cast<T*>(a.cache) + number * page.elements() + (kind == kKeys ? unit / a.maps : unit) * page.head_elements();
    const uint32_t t = pos % M40LLM_PAGE_TOKENS, pad = kind == kValues ? page.v_tiles * 16u : page.k_tiles * 32u;
    T* q = static_cast<T*>(a.queries) + ((size_t)row * a.maps * a.heads + unit) * pad;
#pragma unroll
    for (int i = 0; i < N; ++i) {
        const uint32_t at = W * (lane + 16u * i);            // pads too: zeros
        if (at >= pad) continue;
        if (kind == kQueries) m40_store_columns<T, W>(q + at, y[i]);
        else if (kind == kKeys) m40_store_columns<T, W>(cache + page.key_at(unit % a.maps, t, at), y[i]);
        else {
#pragma unroll
            for (int k = 0; k < W; ++k) cache[page.value_at(t, at + k)] = M40Act<T>::from(y[i][k]);
        }
    }
}
template <class T, int W, int NQ, int NV>
__global__ __launch_bounds__(kThreads) void pair_split_append_kernel(M40llmPairSplit a, M40PairPage page) {
    const uint32_t row = blockIdx.x * 16u + (threadIdx.x >> 4), lane = threadIdx.x & 15u, unit = blockIdx.y;
    if (row >= a.rows) return;           // no barrier below; the 16 lanes of a row stay together
    const uint32_t queries = a.maps * a.heads, keys = a.maps * a.kv_heads;
    if (unit < queries) split_unit<T, W, NQ>(a, page, kQueries, unit, row, lane);
    else if (unit < queries + keys) split_unit<T, W, NQ>(a, page, kKeys, unit - queries, row, lane);
    else split_unit<T, W, NV>(a, page, kValues, unit - queries - keys, row, lane);
}

// A thread a column: the last rows of a portion take their places in the ring.
__global__ __launch_bounds__(kThreads) void conv_state_kernel(const float* __restrict__ proj, size_t ld_proj, uint32_t cols, uint32_t keep,
                                                              float* __restrict__ state, size_t ld_state, const uint32_t* __restrict__ portions,
                                                              const uint32_t* __restrict__ row_pos) {
    const uint32_t row = portions[4 * blockIdx.y], n = portions[4 * blockIdx.y + 1], slot = portions[4 * blockIdx.y + 2];
    const uint32_t c = blockIdx.x * kThreads + threadIdx.x;
    if (n < 2u || c >= cols) return;
    float* s = state + (size_t)slot * keep * ld_state + c;
    const uint32_t first = row_pos[row];
    for (uint32_t i = n > keep ? n - keep : 0u; i < n; ++i) s[(size_t)((first + i) % keep) * ld_state] = proj[(size_t)(row + i) * ld_proj + c];
}

template <class T>
void launch_split(hipStream_t stream, const M40llmPairSplit& s, const M40PairPage& page) {
    const dim3 grid((s.rows + 15u) / 16u, s.maps * s.heads + (s.cache ? (s.maps + 1u) * s.kv_heads : 0u));
    const bool vec = s.dim % 4u == 0 && s.vdim % 4u == 0 && s.ld_proj % 4u == 0 && s.ld_state % 4u == 0 && s.k_offset % 4u == 0 && s.v_offset % 4u == 0 &&
                     m40_aligned16(s.proj) && m40_aligned16(s.conv_state) && m40_aligned16(s.q_conv) && m40_aligned16(s.k_conv) && m40_aligned16(s.v_conv) &&
                     m40_aligned16(s.q_norm) && m40_aligned16(s.k_norm);
    if (!vec) pair_split_append_kernel<T, 1, 16, 16><<<grid, kThreads, 0, stream>>>(s, page);
    else if (s.dim <= 64u && s.vdim <= 64u) pair_split_append_kernel<T, 4, 1, 1><<<grid, kThreads, 0, stream>>>(s, page);
    else if (s.dim <= 64u && s.vdim <= 128u) pair_split_append_kernel<T, 4, 1, 2><<<grid, kThreads, 0, stream>>>(s, page);
    else if (s.dim <= 128u && s.vdim <= 128u) pair_split_append_kernel<T, 4, 2, 2><<<grid, kThreads, 0, stream>>>(s, page);
    else pair_split_append_kernel<T, 4, 4, 4><<<grid, kThreads, 0, stream>>>(s, page);
}

int launched() { return hipGetLastError() == hipSuccess ? 0 : -2; }

}  // namespace

extern "C" {

int m40llm_ext_norm_add_rows_async(M40llmCudaContext* ctx, const M40llmNormAdd* n, uint32_t stream_kind) {
    if (!ctx || !n || !n->x || !n->w || !n->h || (!n->place && (!n->planes || n->n_planes == 0)) ||
        (n->place && (!n->expert_out || !n->weight || n->top == 0)))
        return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    if (n->rows == 0 || n->width == 0 || n->ld_h < n->width || n->ld_h % 32u != 0 || n->act_dtype > 1u || !m40_aligned16(n->h) || (n->h_rows && !m40_aligned16(n->h_rows)))
        return -3;
    const bool vec = n->width % 8u == 0 && m40_aligned16(n->x) && (n->place ? n->ld_expert % 8u == 0 && m40_aligned16(n->expert_out) : n->plane_stride % 4u == 0 && m40_aligned16(n->planes));
    if (n->act_dtype == M40LLM_ACT_F32) {
        if (vec) norm_add_rows_kernel<float, true><<<n->rows, kThreads, 0, stream>>>(*n);
        else norm_add_rows_kernel<float, false><<<n->rows, kThreads, 0, stream>>>(*n);
    } else {
        if (vec) norm_add_rows_kernel<m40_bf16, true><<<n->rows, kThreads, 0, stream>>>(*n);
        else norm_add_rows_kernel<m40_bf16, false><<<n->rows, kThreads, 0, stream>>>(*n);
    }
    return launched();
}

int m40llm_ext_norm_gate_rows_async(M40llmCudaContext* ctx, const void* d_y, uint64_t ld_y, const void* d_w, const void* d_gate, uint64_t ld_gate,
                                    uint32_t rows, uint32_t cols, float eps, void* d_out, uint32_t ld_out, uint32_t act_dtype, uint32_t stream_kind) {
    if (!ctx || !d_y || !d_w || !d_gate || !d_out) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    if (rows == 0 || cols == 0 || ld_out < cols || ld_out % 32u != 0 || ld_y < cols || ld_gate < cols || act_dtype > 1u || !m40_aligned16(d_out)) return -3;
    const float *y = static_cast<const float*>(d_y), *w = static_cast<const float*>(d_w), *g = static_cast<const float*>(d_gate);
    const bool vec = cols % 8u == 0 && ld_y % 4u == 0 && ld_gate % 4u == 0 && m40_aligned16(d_y) && m40_aligned16(d_gate);
    auto go = [&](auto kernel, auto* out) { kernel<<<rows, kThreads, 0, stream>>>(y, (size_t)ld_y, w, g, (size_t)ld_gate, rows, cols, eps, out, ld_out); };
    if (act_dtype == M40LLM_ACT_F32) {
        if (vec) go(norm_gate_rows_kernel<float, true>, static_cast<float*>(d_out));
        else go(norm_gate_rows_kernel<float, false>, static_cast<float*>(d_out));
    } else {
        if (vec) go(norm_gate_rows_kernel<m40_bf16, true>, static_cast<m40_bf16*>(d_out));
        else go(norm_gate_rows_kernel<m40_bf16, false>, static_cast<m40_bf16*>(d_out));
    }
    return launched();
}

uint64_t m40llm_ext_pair_page_elements(uint32_t maps, uint32_t kv_heads, uint32_t dim, uint32_t vdim) { return M40PairPage(maps, kv_heads, dim, vdim).elements(); }

int m40llm_ext_pair_split_append_async(M40llmCudaContext* ctx, const M40llmPairSplit* s, uint32_t stream_kind) {
    if (!ctx || !s || !s->proj || !s->q_norm || !s->queries || !s->row_slot || !s->row_pos || !s->row_back) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    if (s->rows == 0 || s->act_dtype > 1u || s->maps == 0 || s->maps > 2u || s->heads == 0 || s->kv_heads == 0 || s->heads % s->kv_heads != 0 || s->dim == 0 ||
        s->dim > M40LLM_PAIR_MOST_DIM || s->vdim == 0 || s->vdim > M40LLM_PAIR_MOST_DIM || s->maps * (s->heads + (uint64_t)s->kv_heads) + s->kv_heads > 65535u)
        return -3;
    const uint64_t cols = s->cache ? (uint64_t)s->v_offset + (uint64_t)s->kv_heads * s->vdim : (uint64_t)s->maps * s->heads * s->dim;
    if (s->ld_proj < cols) return -3;
    if (s->taps && (!s->q_conv || (s->taps > 1u && (!s->conv_state || s->ld_state < cols)))) return -4;
    if (s->cache && (!s->k_norm || !s->page_table || s->k_offset < s->maps * s->heads * s->dim || s->v_offset < s->k_offset + s->maps * s->kv_heads * s->dim ||
                     (s->taps && (!s->k_conv || !s->v_conv))))
        return -4;
    const M40PairPage page(s->maps, s->kv_heads, s->dim, s->vdim);
    if (s->act_dtype == M40LLM_ACT_F32) launch_split<float>(stream, *s, page);
    else launch_split<m40_bf16>(stream, *s, page);
    return launched();
}

int m40llm_ext_conv_state_async(M40llmCudaContext* ctx, const void* d_proj, uint64_t ld_proj, uint32_t cols, uint32_t taps, void* d_state, uint64_t ld_state,
                                const uint32_t* d_portions, const uint32_t* d_row_pos, uint32_t n_portions, uint32_t stream_kind) {
    if (!ctx || !d_proj || !d_state || !d_portions || !d_row_pos) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    if (cols == 0 || taps < 2u || ld_proj < cols || ld_state < cols || n_portions == 0 || n_portions > 65535u) return -3;
    conv_state_kernel<<<dim3((cols + kThreads - 1) / kThreads, n_portions), kThreads, 0, stream>>>(static_cast<const float*>(d_proj), (size_t)ld_proj, cols,
                                                                                                  taps - 1u, static_cast<float*>(d_state), (size_t)ld_state, d_portions, d_row_pos);
    return launched();
}

}  // extern "C"
