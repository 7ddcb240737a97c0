// Row-wise steps of layered decoders: embedding (token, token pair, position), norms, rotation angles, and the step between a latent
// attention's projections and its attention (norms of the two latents, rotation, cache append).
#include "packed_gemm.hpp"

#include <type_traits>

namespace {

constexpr int kThreads = 256;

template <class T>
__global__ __launch_bounds__(kThreads) void embed_tokens_kernel(M40llmEmbedTokens e) {
    const uint32_t row = m40_tile_row(blockIdx.x, e.rows), width = e.width;
    uint32_t tok = e.tokens[row];
    tok = tok < e.vocab ? tok : e.vocab - 1u;
    const uint16_t* a = static_cast<const uint16_t*>(e.table) + (size_t)tok * width;
    const uint16_t *b = nullptr, *c = nullptr;
    if (e.pair_table) {
        const uint32_t p = e.prev[row];
        const uint32_t r = p == 0xffffffffu ? e.buckets : (uint32_t)(((uint64_t)p * e.mul_prev + (uint64_t)tok * e.mul_cur) % e.buckets);
        b = static_cast<const uint16_t*>(e.pair_table) + (size_t)r * width;
    }
    if (e.pos_table) {
        const uint32_t p = e.positions[row];
        c = static_cast<const uint16_t*>(e.pos_table) + (size_t)(p < e.n_positions ? p : e.n_positions - 1u) * width;
    }
    float* out = static_cast<float*>(e.x) + (size_t)row * width;
    T* h = static_cast<T*>(e.h);
    if (width % 8u == 0) {
        for (uint32_t i = threadIdx.x; i < width / 8u; i += kThreads) {
            m40_f32x8 v = __builtin_convertvector(reinterpret_cast<const m40_bf16x8*>(a)[i], m40_f32x8) * e.scale;
            if (b) v += __builtin_convertvector(reinterpret_cast<const m40_bf16x8*>(b)[i], m40_f32x8);
            if (c) v += __builtin_convertvector(reinterpret_cast<const m40_bf16x8*>(c)[i], m40_f32x8);
            reinterpret_cast<m40_f32x8*>(out)[i] = v;
            if (h) {
                T* o = h + m40_packed_at(row, i * 8u, e.ld_h >> 5);
                m40_store4<T>(o, m40_float4{v[0], v[1], v[2], v[3]});
                m40_store4<T>(o + 4, m40_float4{v[4], v[5], v[6], v[7]});
            }
        }
    } else {
        for (uint32_t i = threadIdx.x; i < width; i += kThreads) {
            float v = m40_bf16_bits(a[i]) * e.scale;
            if (b) v += m40_bf16_bits(b[i]);
            if (c) v += m40_bf16_bits(c[i]);
            out[i] = v;
            if (h) h[m40_packed_at(row, i, e.ld_h >> 5)] = M40Act<T>::from(v);
        }
    }
    if (h)
        for (uint32_t i = width + threadIdx.x; i < e.ld_h; i += kThreads) h[m40_packed_at(row, i, e.ld_h >> 5)] = M40Act<T>::from(0.0f);
}

// sum over the workgroup, the same bits in every thread
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

// A thread takes groups of eight neighbouring elements: 16-byte pieces of a packed tile.  RMS: the mean stays where it is.
template <class T, bool VEC, bool RMS>
__global__ __launch_bounds__(kThreads) void layer_norm_rows_kernel(float* __restrict__ x, const float* __restrict__ planes, uint32_t n_planes,
                                                                   size_t plane_stride, const float* __restrict__ w,
                                                                   const uint32_t* __restrict__ row_index, uint32_t width, float eps,
                                                                   T* __restrict__ out, uint32_t ld_out) {
    __shared__ float scratch[kThreads / 64];
    constexpr uint32_t kGroups = 2;      // groups a thread keeps in registers (width up to 4096); beyond, they are read again
    const uint32_t out_row = m40_tile_row(blockIdx.x, gridDim.x);
    const size_t at = (size_t)(row_index ? row_index[out_row] : out_row) * width;
    const uint32_t groups = ld_out / 8u;
    auto load = [&](uint32_t g, float (&v)[8]) __attribute__((always_inline)) {
        auto add = [&](const float* src, bool first) __attribute__((always_inline)) {
            if (VEC) {
                const float4 a = reinterpret_cast<const float4*>(src + g * 8u)[0], b = reinterpret_cast<const float4*>(src + g * 8u)[1];
                const float t[8] = {a.x, a.y, a.z, a.w, b.x, b.y, b.z, b.w};
#pragma unroll
                for (int i = 0; i < 8; ++i) v[i] = first ? t[i] : v[i] + t[i];
            } else {
#pragma unroll
                for (uint32_t i = 0; i < 8; ++i) {
                    const float t = g * 8u + i < width ? src[g * 8u + i] : 0.0f;
                    v[i] = first ? t : v[i] + t;
                }
            }
        };
        if (g * 8u >= width) {
#pragma unroll
            for (int i = 0; i < 8; ++i) v[i] = 0.0f;
            return;
        }
        add(x + at, true);
        for (uint32_t p = 0; p < n_planes; ++p) add(planes + p * plane_stride + at, false);
    };
    auto keep_sum = [&](uint32_t g, const float (&v)[8]) __attribute__((always_inline)) {      // x takes the planes' sums
        if (n_planes == 0 || row_index || g * 8u >= width) return;
        if (VEC) {
            reinterpret_cast<float4*>(x + at + g * 8u)[0] = make_float4(v[0], v[1], v[2], v[3]);
            reinterpret_cast<float4*>(x + at + g * 8u)[1] = make_float4(v[4], v[5], v[6], v[7]);
        } else {
#pragma unroll
            for (uint32_t i = 0; i < 8; ++i)
                if (g * 8u + i < width) x[at + g * 8u + i] = v[i];
        }
    };
    float keep[kGroups][8];
    float s = 0.0f;
    auto sum8 = [&](const float (&v)[8]) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < 8; ++i) s += v[i];
    };
    float mean = 0.0f, q = 0.0f;
    auto sq8 = [&](uint32_t g, const float (&v)[8]) __attribute__((always_inline)) {
#pragma unroll
        for (uint32_t i = 0; i < 8; ++i) {
            const float d = g * 8u + i < width ? v[i] - mean : 0.0f;
            q = fmaf(d, d, q);
        }
    };
    float inv = 0.0f;
    auto store = [&](uint32_t g, const float (&v)[8]) __attribute__((always_inline)) {
        T* o = out + m40_packed_at(out_row, g * 8u, ld_out >> 5);
        m40_float4 lo, hi;
#pragma unroll
        for (uint32_t i = 0; i < 4; ++i) {
            lo[i] = g * 8u + i < width ? (v[i] - mean) * inv * w[g * 8u + i] : 0.0f;
            hi[i] = g * 8u + 4u + i < width ? (v[4 + i] - mean) * inv * w[g * 8u + 4u + i] : 0.0f;
        }
        m40_store4<T>(o, lo);
        m40_store4<T>(o + 4, hi);
    };
#pragma unroll
    for (uint32_t j = 0; j < kGroups; ++j) {
        const uint32_t g = threadIdx.x + j * kThreads;
        load(g < groups ? g : groups, keep[j]);          // past the end: zeros
        if (g < groups) keep_sum(g, keep[j]);
        sum8(keep[j]);
    }
    for (uint32_t g = threadIdx.x + kGroups * kThreads; g < groups; g += kThreads) {
        float v[8];
        load(g, v);
        sum8(v);
    }
    if (!RMS) mean = block_sum(s, scratch) / (float)width;
#pragma unroll
    for (uint32_t j = 0; j < kGroups; ++j) sq8(threadIdx.x + j * kThreads, keep[j]);
    for (uint32_t g = threadIdx.x + kGroups * kThreads; g < groups; g += kThreads) {
        float v[8];
        load(g, v);
        sq8(g, v);
    }
    inv = 1.0f / sqrtf(block_sum(q, scratch) / (float)width + eps);
#pragma unroll
    for (uint32_t j = 0; j < kGroups; ++j) {
        const uint32_t g = threadIdx.x + j * kThreads;
        if (g < groups) store(g, keep[j]);
    }
    for (uint32_t g = threadIdx.x + kGroups * kThreads; g < groups; g += kThreads) {
        float v[8];
        load(g, v);
        store(g, v);
        keep_sum(g, v);
    }
}

__global__ __launch_bounds__(kThreads) void rotation_angles_kernel(const uint32_t* __restrict__ positions, const double* __restrict__ freq,
                                                                   uint32_t rows, uint32_t pairs, uint32_t ld_pairs, float magnitude,
                                                                   float2* __restrict__ angles) {
    const size_t i = (size_t)blockIdx.x * kThreads + threadIdx.x;
    if (i >= (size_t)rows * ld_pairs) return;
    const uint32_t row = (uint32_t)(i / ld_pairs), p = (uint32_t)(i % ld_pairs);
    if (p >= pairs) {
        angles[i] = make_float2(1.0f, 0.0f);
        return;
    }
    double s, c;
    sincos((double)positions[row] * freq[p], &s, &c);
    angles[i] = make_float2((float)(c * (double)magnitude), (float)(s * (double)magnitude));
}

template <class T>
__global__ __launch_bounds__(kThreads) void latent_split_append_kernel(M40llmLatentSplit a) {
    __shared__ float scratch[kThreads / 64];
    const uint32_t row = m40_tile_row(blockIdx.x, a.rows), tid = threadIdx.x;
    const float* src = static_cast<const float*>(a.proj) + (size_t)row * a.ld_proj;
    float s = 0.0f;
    for (uint32_t i = tid; i < a.q_rank; i += kThreads) s = fmaf(src[i], src[i], s);
    const float q_inv = 1.0f / sqrtf(block_sum(s, scratch) / (float)a.q_rank + a.eps);
    T* cq = static_cast<T*>(a.cq);
    const float* qw = static_cast<const float*>(a.q_norm);
    for (uint32_t i = tid; i < a.ld_cq; i += kThreads) cq[m40_packed_at(row, i, a.ld_cq >> 5)] = M40Act<T>::from(i < a.q_rank ? src[i] * q_inv * qw[i] : 0.0f);
    if (!a.cache) return;
    const float* kv = src + a.kv_offset;
    s = 0.0f;
    for (uint32_t i = tid; i < a.kv_rank; i += kThreads) s = fmaf(kv[i], kv[i], s);
    const float kv_inv = 1.0f / sqrtf(block_sum(s, scratch) / (float)a.kv_rank + a.eps);
    const float* kw = static_cast<const float*>(a.kv_norm);
    const uint32_t pos = a.row_pos[row], page = a.page_table[(size_t)a.row_slot[row] * a.max_pages + pos / M40LLM_PAGE_TOKENS];
    const uint32_t t = pos % M40LLM_PAGE_TOKENS, k_tiles = a.entry_width / 32u;
    T* entry = static_cast<T*>(a.cache) + (size_t)page * M40LLM_PAGE_TOKENS * a.entry_width + (size_t)(t / 16u) * k_tiles * kM40Tile;
    auto place = [&](uint32_t k) { return (size_t)(k / 32u) * kM40Tile + m40_tile_offset(t % 16u, k % 32u); };
    for (uint32_t i = tid; i < a.latent_pad; i += kThreads)
        entry[place(i)] = M40Act<T>::from(i < a.kv_rank ? kv[i] * kv_inv * kw[i] : 0.0f);
    const float* rot = src + a.rot_offset;
    const float2* ang = static_cast<const float2*>(a.angles) + (size_t)row * a.rot_half;
    for (uint32_t i = tid; i < a.entry_width - a.latent_pad; i += kThreads) {
        float y = 0.0f;
        if (i < a.rot_dim) {
            const float2 cs = ang[i >> 1];
            const float u = rot[i & ~1u], v = (i | 1u) < a.rot_dim ? rot[i | 1u] : 0.0f;
            y = (i & 1u) ? fmaf(v, cs.x, u * cs.y) : fmaf(u, cs.x, -(v * cs.y));
        }
        entry[place(a.latent_pad + i)] = M40Act<T>::from(y);
    }
}

struct Top2 {
    float best, second;
    uint32_t at, unused;
};
__device__ __forceinline__ void top2_join(Top2& a, const Top2& b) {       // the lower index of equal logits
    const bool take = b.best > a.best || (b.best == a.best && b.at < a.at);
    a.second = take ? fmaxf(a.best, b.second) : fmaxf(a.second, b.best);
    a.best = take ? b.best : a.best;
    a.at = take ? b.at : a.at;
}
__device__ __forceinline__ Top2 top2_wave(Top2 t) {
#pragma unroll
    for (int d = 1; d < 64; d *= 2) top2_join(t, Top2{__shfl_xor(t.best, d), __shfl_xor(t.second, d), (uint32_t)__shfl_xor((int)t.at, d), 0u});
    return t;
}
__global__ __launch_bounds__(kThreads) void top2_parts_kernel(const float* __restrict__ logits, uint32_t vocab, Top2* __restrict__ parts) {
    __shared__ Top2 wave_top[kThreads / 64];
    const uint32_t per = (vocab + M40LLM_TOP2_PARTS - 1u) / M40LLM_TOP2_PARTS, begin = blockIdx.x * per;
    const uint32_t end = begin + per < vocab ? begin + per : vocab;
    const float* row = logits + (size_t)blockIdx.y * vocab;
    Top2 t{-INFINITY, -INFINITY, 0xffffffffu, 0u};
    for (uint32_t i = begin + threadIdx.x; i < end; i += kThreads) top2_join(t, Top2{row[i], -INFINITY, i, 0u});
    t = top2_wave(t);
    if ((threadIdx.x & 63u) == 0u) wave_top[threadIdx.x >> 6] = t;
    __syncthreads();
    if (threadIdx.x != 0u) return;
    for (int w = 1; w < kThreads / 64; ++w) top2_join(t, wave_top[w]);
    parts[blockIdx.y * M40LLM_TOP2_PARTS + blockIdx.x] = t;
}

// a wave a row
__global__ __launch_bounds__(kThreads) void advance_rows_kernel(const Top2* __restrict__ parts, uint32_t rows,
                                                                uint32_t* __restrict__ tokens, uint32_t* __restrict__ prev,
                                                                uint32_t* __restrict__ positions, uint32_t* __restrict__ state,
                                                                uint32_t* __restrict__ ids, float* __restrict__ gaps, uint32_t capacity) {
    const uint32_t step = state[0], lane = threadIdx.x & 63u;
    __syncthreads();
    for (uint32_t r = threadIdx.x >> 6; r < rows; r += kThreads / 64) {
        Top2 t = lane < M40LLM_TOP2_PARTS ? parts[r * M40LLM_TOP2_PARTS + lane] : Top2{-INFINITY, -INFINITY, 0xffffffffu, 0u};
        t = top2_wave(t);
        if (lane != 0u) continue;
        const uint32_t next = t.at == 0xffffffffu ? 0u : t.at;          // no comparable logit
        if (step < capacity) {
            ids[(size_t)r * capacity + step] = next;
            gaps[(size_t)r * capacity + step] = t.best - t.second;
        }
        prev[r] = tokens[r];
        tokens[r] = next;
        positions[r] += 1u;
    }
    if (threadIdx.x == 0u) state[0] = step + 1u;
}

int launched() { return hipGetLastError() == hipSuccess ? 0 : -2; }

}  // namespace

extern "C" {

int m40llm_ext_embed_tokens_async(M40llmCudaContext* ctx, const M40llmEmbedTokens* e, uint32_t stream_kind) {
    if (!ctx || !e || !e->table || !e->tokens || !e->x || (e->pair_table && !e->prev) || (e->pos_table && !e->positions)) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    if (e->rows == 0 || e->vocab == 0 || e->width == 0 || e->act_dtype > 1u || (e->pair_table && e->buckets == 0) || (e->pos_table && e->n_positions == 0) ||
        (e->h && (e->ld_h < e->width || e->ld_h % 32u != 0 || !m40_aligned16(e->h))))
        return -3;
    if (e->act_dtype == M40LLM_ACT_F32) embed_tokens_kernel<float><<<e->rows, kThreads, 0, stream>>>(*e);
    else embed_tokens_kernel<m40_bf16><<<e->rows, kThreads, 0, stream>>>(*e);
    return launched();
}

int m40llm_ext_embed_pairs_async(M40llmCudaContext* ctx, const void* d_table, const void* d_pairs, const uint32_t* d_tokens,
                                 const uint32_t* d_prev, uint32_t rows, uint32_t vocab, uint32_t width, uint32_t buckets,
                                 uint32_t mul_prev, uint32_t mul_cur, void* d_x, uint32_t stream_kind) {
    M40llmEmbedTokens e{};
    e.rows = rows; e.vocab = vocab; e.width = width;
    e.table = d_table; e.pair_table = d_pairs; e.tokens = d_tokens; e.prev = d_prev;
    e.buckets = buckets; e.mul_prev = mul_prev; e.mul_cur = mul_cur;
    e.scale = 1.0f;
    e.x = d_x;
    return m40llm_ext_embed_tokens_async(ctx, &e, stream_kind);
}

int m40llm_ext_norm_rows_async(M40llmCudaContext* ctx, uint32_t norm_kind, void* d_x, const void* d_planes, uint32_t n_planes, uint64_t plane_stride,
                               const void* d_w, const uint32_t* d_row_index, uint32_t rows, uint32_t width, float eps, void* d_out,
                               uint32_t ld_out, uint32_t act_dtype, uint32_t stream_kind) {
    if (!ctx || !d_x || !d_w || !d_out || (n_planes && !d_planes)) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    if (norm_kind > M40LLM_NORM_RMS || rows == 0 || width == 0 || ld_out < width || ld_out % 32u != 0 || act_dtype > 1u || !m40_aligned16(d_out)) return -3;
    float* x = static_cast<float*>(d_x);
    const float *w = static_cast<const float*>(d_w), *p = static_cast<const float*>(d_planes);
    const bool vec = width % 8u == 0 && plane_stride % 4u == 0 && m40_aligned16(d_x) && (!n_planes || m40_aligned16(d_planes));
    auto go = [&](auto kernel, auto* out) { kernel<<<rows, kThreads, 0, stream>>>(x, p, n_planes, (size_t)plane_stride, w, d_row_index, width, eps, out, ld_out); };
    auto pick = [&](auto* out, auto rms) {
        typedef std::remove_reference_t<decltype(*out)> T;
        constexpr bool kRms = decltype(rms)::value;
        if (vec) go(layer_norm_rows_kernel<T, true, kRms>, out);
        else go(layer_norm_rows_kernel<T, false, kRms>, out);
    };
    auto kind = [&](auto* out) {
        if (norm_kind == M40LLM_NORM_RMS) pick(out, std::true_type());
        else pick(out, std::false_type());
    };
    if (act_dtype == M40LLM_ACT_F32) kind(static_cast<float*>(d_out));
    else kind(static_cast<m40_bf16*>(d_out));
    return launched();
}

int m40llm_ext_layer_norm_rows_async(M40llmCudaContext* ctx, void* d_x, const void* d_planes, uint32_t n_planes, uint64_t plane_stride,
                                     const void* d_w, const uint32_t* d_row_index, uint32_t rows, uint32_t width, float eps, void* d_out,
                                     uint32_t ld_out, uint32_t act_dtype, uint32_t stream_kind) {
    return m40llm_ext_norm_rows_async(ctx, M40LLM_NORM_LAYER, d_x, d_planes, n_planes, plane_stride, d_w, d_row_index, rows, width, eps, d_out, ld_out,
                                      act_dtype, stream_kind);
}

int m40llm_ext_rotation_angles_async(M40llmCudaContext* ctx, const uint32_t* d_positions, uint32_t rows, const double* d_freq, uint32_t pairs,
                                     uint32_t ld_pairs, float magnitude, void* d_angles, uint32_t stream_kind) {
    if (!ctx || !d_positions || !d_freq || !d_angles) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    if (rows == 0 || ld_pairs == 0 || pairs > ld_pairs) return -3;
    const size_t n = (size_t)rows * ld_pairs;
    rotation_angles_kernel<<<(unsigned)((n + kThreads - 1) / kThreads), kThreads, 0, stream>>>(d_positions, d_freq, rows, pairs, ld_pairs,
                                                                                              magnitude, static_cast<float2*>(d_angles));
    return launched();
}

int m40llm_ext_latent_split_append_async(M40llmCudaContext* ctx, const M40llmLatentSplit* s, uint32_t stream_kind) {
    if (!ctx || !s || !s->proj || !s->q_norm || !s->cq) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    if (s->rows == 0 || s->q_rank == 0 || s->ld_cq < s->q_rank || s->ld_cq % 32u != 0 || s->act_dtype > 1u) return -3;
    if (s->cache && (!s->kv_norm || !s->angles || !s->row_slot || !s->row_pos || !s->page_table || s->kv_rank == 0 ||
                     s->latent_pad < s->kv_rank || s->latent_pad % 32u != 0 || s->entry_width % 32u != 0 ||
                     s->entry_width < s->latent_pad + s->rot_dim || s->rot_half * 2u < s->rot_dim))
        return -3;
    if (s->act_dtype == M40LLM_ACT_F32) latent_split_append_kernel<float><<<s->rows, kThreads, 0, stream>>>(*s);
    else latent_split_append_kernel<m40_bf16><<<s->rows, kThreads, 0, stream>>>(*s);
    return launched();
}

int m40llm_ext_top2_parts_async(M40llmCudaContext* ctx, const void* d_logits, uint32_t rows, uint32_t vocab, void* d_parts, uint32_t stream_kind) {
    if (!ctx || !d_logits || !d_parts) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    if (rows == 0 || rows > 65535u || vocab == 0 || !m40_aligned16(d_parts)) return -3;
    top2_parts_kernel<<<dim3(M40LLM_TOP2_PARTS, rows), kThreads, 0, stream>>>(static_cast<const float*>(d_logits), vocab, static_cast<Top2*>(d_parts));
    return launched();
}

int m40llm_ext_advance_rows_async(M40llmCudaContext* ctx, const void* d_parts, uint32_t rows, uint32_t* d_tokens, uint32_t* d_prev,
                                  uint32_t* d_positions, uint32_t* d_state, uint32_t* d_ids, float* d_gaps, uint32_t capacity,
                                  uint32_t stream_kind) {
    if (!ctx || !d_parts || !d_tokens || !d_prev || !d_positions || !d_state || !d_ids || !d_gaps) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    if (rows == 0 || !m40_aligned16(d_parts)) return -3;
    advance_rows_kernel<<<1, kThreads, 0, stream>>>(static_cast<const Top2*>(d_parts), rows, d_tokens, d_prev, d_positions, d_state, d_ids, d_gaps,
                                                    capacity);
    return launched();
}

}  // extern "C"
