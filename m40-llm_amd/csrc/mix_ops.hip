// Row-wise steps of pre-norm layers.
//
// token_mix_kernel         each row mixed with the one before it in several proportions
// space_split_kernel       state space layers: short convolution with bias and silu, rows as the recurrence reads them.  A workgroup takes 16 rows
//                          of one head
// gate_group_norm_kernel   a gate, then an RMS norm over each of several parts of a row; a wave or a workgroup a part
// poly_norm_rows_kernel,   polynomial whose powers are each divided by their root mean square over the row, in place: a workgroup a row, or (many
// poly_norm_tiles_kernel   rows) a workgroup a tile of 16 rows, which reads and writes whole kilobytes
#include "short_conv.hpp"

namespace {

constexpr uint32_t kThreads = 256;

// columns at .. at + 7 of a row of `cols`, zero past them
template <bool VEC>
__device__ __forceinline__ void load8(const float* row, uint32_t at, uint32_t cols, float (&v)[8]) {
    if (VEC) {
        const float4 a = reinterpret_cast<const float4*>(row + at)[0], b = reinterpret_cast<const float4*>(row + at)[1];
        v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w; v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
    } else {
#pragma unroll
        for (uint32_t i = 0; i < 8; ++i) v[i] = at + i < cols ? row[at + i] : 0.0f;
    }
}
template <class T>
__device__ __forceinline__ void store8(T* p, const float (&v)[8]) {
    m40_store4<T>(p, m40_float4{v[0], v[1], v[2], v[3]});
    m40_store4<T>(p + 4, m40_float4{v[4], v[5], v[6], v[7]});
}

// ---- token mix: workgroups 0 .. rows - 1 take the rows that are not a portion's first, the others a portion's first row and its state
template <class T>
__global__ __launch_bounds__(kThreads) void token_mix_kernel(M40llmTokenMix a) {
    const bool inner = blockIdx.x < a.rows;
    const uint32_t* portion = inner ? nullptr : a.portions + 4 * (blockIdx.x - a.rows);
    const uint32_t row = inner ? m40_tile_row(blockIdx.x, a.rows) : portion[0];
    if (inner && (a.row_back[row] & 0x7fffffffu) == 0u) return;
    const T* h = static_cast<const T*>(a.h) + (size_t)row * a.ld;
    float* state = inner ? nullptr : static_cast<float*>(a.state) + (size_t)portion[2] * a.ld;
    const bool fresh = !inner && a.row_pos[row] == 0u;
    const T* last = inner ? nullptr : static_cast<const T*>(a.h) + (size_t)(row + portion[1] - 1u) * a.ld;
    T* out = static_cast<T*>(a.out);
    const float* mu = static_cast<const float*>(a.mu);
    const uint32_t tiles = a.mixes * a.ld / 32u;
    for (uint32_t c = threadIdx.x * 8u; c < a.ld; c += kThreads * 8u) {
        const typename M40Act<T>::vec8 now = M40Act<T>::load8(h + c);
        float x[8], d[8];
        if (inner) {
            const typename M40Act<T>::vec8 before = M40Act<T>::load8(h - a.ld + c);
#pragma unroll
            for (int i = 0; i < 8; ++i) d[i] = M40Act<T>::to(before[i]);
        } else {
            load8<true>(state, c, a.ld, d);
            const typename M40Act<T>::vec8 next = M40Act<T>::load8(last + c);
            float keep[8];
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                keep[i] = M40Act<T>::to(next[i]);
                d[i] = fresh ? 0.0f : d[i];
            }
            store8<float>(state + c, keep);
        }
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            x[i] = M40Act<T>::to(now[i]);
            d[i] -= x[i];
        }
#pragma unroll 5
        for (uint32_t m = 0; m < a.mixes; ++m) {
            float w[8], y[8];
            load8<true>(mu + (size_t)m * a.ld, c, a.ld, w);
#pragma unroll
            for (int i = 0; i < 8; ++i) y[i] = fmaf(d[i], w[i], x[i]);
            store8<T>(out + m40_packed_at(row, m * a.ld + c, tiles), y);
        }
    }
}

// ---- convolution, silu
template <class T, int W, int N>
__global__ __launch_bounds__(kThreads) void space_split_kernel(M40llmSpaceSplit a) {
    const uint32_t row = blockIdx.x * 16u + (threadIdx.x >> 4), lane = threadIdx.x & 15u;
    if (row >= a.rows) return;               // no barrier below; the 16 lanes of a row stay together
    const uint32_t d_pad = (a.dim + 31u) & ~31u, v_pad = (a.vdim + 31u) & ~31u, unit = blockIdx.y, shared = a.kv_heads * a.dim, values = a.heads * a.vdim;
    // units: heads of queries, of keys, of values; columns: values, keys, queries
    const bool value = unit >= 2u * a.kv_heads, key = !value && unit >= a.kv_heads;
    const uint32_t n = value ? a.vdim : a.dim, pad = value ? v_pad : d_pad;
    const uint32_t col0 = value ? (unit - 2u * a.kv_heads) * a.vdim : key ? values + (unit - a.kv_heads) * a.dim : values + shared + unit * a.dim;
    const uint32_t to = value ? 2u * a.kv_heads * d_pad + (unit - 2u * a.kv_heads) * v_pad : unit * d_pad;
    const uint32_t keep = a.taps - 1u, slot = a.row_slot[row];
    const M40ConvRow r{static_cast<const float*>(a.proj) + (size_t)row * a.ld_proj + col0, (size_t)a.ld_proj, static_cast<const float*>(a.conv) + col0, values + 2u * shared, a.taps,
                       keep ? static_cast<float*>(a.conv_state) + (size_t)slot * keep * a.ld_state + col0 : nullptr, (size_t)a.ld_state, a.row_pos[row], a.row_back[row]};
    float y[N][W];
    m40_short_conv<W, N>(r, n, lane, y);
    const float* bias = static_cast<const float*>(a.bias) + col0;
    T* out = static_cast<T*>(a.out);
#pragma unroll
    for (int i = 0; i < N; ++i) {
        const uint32_t at = W * (lane + 16u * i);
        if (at >= pad) continue;
        const M40Columns<W> b = m40_load_columns<W>(bias + (at < n ? at : 0u));
#pragma unroll
        for (int k = 0; k < W; ++k) y[i][k] = at < n ? m40_silu(y[i][k] + b.v[k]) : 0.0f;
        m40_store_columns<T, W>(out + m40_packed_at(row, to + at, (uint32_t)(a.ld_out >> 5)), y[i]);
    }
}

// ---- gate and norm over parts.  TEAM threads a part.
struct GroupNormArgs {
    const float *y, *gate, *w;
    size_t ld_y, ld_gate;
    uint32_t rows, cols, groups, part;
    float eps;
    void* out;
    uint32_t ld_out;
};
template <class T, uint32_t TEAM, bool VEC>
__global__ __launch_bounds__(kThreads) void gate_group_norm_kernel(GroupNormArgs a) {
    __shared__ float scratch[kThreads / 64];
    constexpr uint32_t kKeep = 2;            // groups of eight columns a thread keeps in registers
    const uint32_t row = m40_tile_row(blockIdx.x, a.rows), lane = threadIdx.x % TEAM, group = blockIdx.y * (kThreads / TEAM) + threadIdx.x / TEAM;
    const bool live = group < a.groups;
    const uint32_t first = (live ? group : 0u) * a.part;
    const float *y = a.y + (size_t)row * a.ld_y + first, *z = a.gate + (size_t)row * a.ld_gate + first, *w = a.w + first;
    auto gated = [&](uint32_t c, float (&u)[8]) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < 8; ++i) u[i] = 0.0f;
        if (!live || c >= a.part) return;
        float g[8];
        load8<VEC>(y, c, a.part, u);
        load8<VEC>(z, c, a.part, g);
#pragma unroll
        for (int i = 0; i < 8; ++i) u[i] *= m40_silu(g[i]);
    };
    float kept[kKeep][8], q = 0.0f;
#pragma unroll
    for (uint32_t j = 0; j < kKeep; ++j) {
        gated((lane + j * TEAM) * 8u, kept[j]);
#pragma unroll
        for (int i = 0; i < 8; ++i) q = fmaf(kept[j][i], kept[j][i], q);
    }
    for (uint32_t c = (lane + kKeep * TEAM) * 8u; c < a.part; c += TEAM * 8u) {
        float u[8];
        gated(c, u);
#pragma unroll
        for (int i = 0; i < 8; ++i) q = fmaf(u[i], u[i], q);
    }
    q = m40_sum64(q);
    if (TEAM > 64) {
        if ((threadIdx.x & 63u) == 0u) scratch[threadIdx.x >> 6] = q;
        __syncthreads();
        q = scratch[0] + scratch[1] + scratch[2] + scratch[3];
    }
    if (!live) return;
    const float inv = 1.0f / sqrtf(q / (float)a.part + a.eps);
    T* out = static_cast<T*>(a.out);
    const uint32_t tiles = a.ld_out >> 5;
    auto finish = [&](uint32_t c, const float (&u)[8]) __attribute__((always_inline)) {
        if (c >= a.part) return;
        float v[8];
        load8<VEC>(w, c, a.part, v);
#pragma unroll
        for (int i = 0; i < 8; ++i) v[i] *= u[i] * inv;
        if (VEC) {
            store8<T>(out + m40_packed_at(row, first + c, tiles), v);
        } else {
#pragma unroll
            for (uint32_t i = 0; i < 8; ++i)
                if (c + i < a.part) out[m40_packed_at(row, first + c + i, tiles)] = M40Act<T>::from(v[i]);
        }
    };
#pragma unroll
    for (uint32_t j = 0; j < kKeep; ++j) finish((lane + j * TEAM) * 8u, kept[j]);
    for (uint32_t c = (lane + kKeep * TEAM) * 8u; c < a.part; c += TEAM * 8u) {
        float u[8];
        gated(c, u);
        finish(c, u);
    }
    if (group + 1u == a.groups)              // past the last part: zeros
        for (uint32_t c = a.cols + lane; c < a.ld_out; c += TEAM) out[m40_packed_at(row, c, tiles)] = M40Act<T>::from(0.0f);
}

// ---- normed polynomial
struct PolySums {
    float s2 = 0.0f, s4 = 0.0f, s6 = 0.0f;
    __device__ __forceinline__ void take(float z) {
        const float z2 = z * z, z4 = z2 * z2;
        s2 += z2;
        s4 = fmaf(z2, z2, s4);
        s6 = fmaf(z4, z2, s6);
    }
};
struct PolyFactors {
    float f1, f2, f3, e;
    __device__ __forceinline__ PolyFactors(const PolySums& s, const float* act, uint32_t cols, float eps) {
        const float n = 1.0f / (float)cols;
        f1 = act[0] / sqrtf(s.s2 * n + eps);
        f2 = act[1] / sqrtf(s.s4 * n + eps);
        f3 = act[2] / sqrtf(s.s6 * n + eps);
        e = act[3];
    }
    __device__ __forceinline__ float operator()(float z) const { return fmaf(z, fmaf(z, fmaf(z, f3, f2), f1), e); }
};
template <class T>
__device__ __forceinline__ void poly_store(T* p, const typename M40Act<T>::vec8& z, uint32_t col, uint32_t cols, const PolyFactors& f) {
    float y[8];
#pragma unroll
    for (uint32_t i = 0; i < 8; ++i) y[i] = col + i < cols ? f(M40Act<T>::to(z[i])) : 0.0f;
    store8<T>(p, y);
}

template <class T>
__global__ __launch_bounds__(kThreads) void poly_norm_rows_kernel(T* __restrict__ z, uint32_t ld, const float* __restrict__ act, uint32_t rows, uint32_t cols, float eps) {
    __shared__ float part[3][kThreads / 64];
    typedef typename M40Act<T>::vec8 vec8;
    constexpr uint32_t kKeep = 6;
    const uint32_t row = m40_tile_row(blockIdx.x, rows), tid = threadIdx.x, tiles = ld >> 5;
    // columns past cols are zero already: they add nothing
    auto at = [&](uint32_t g) { return z + m40_packed_at(row, g * 8u, tiles); };
    const uint32_t groups = ld / 8u;
    vec8 kept[kKeep];
    PolySums s;
#pragma unroll
    for (uint32_t j = 0; j < kKeep; ++j) {
        const uint32_t g = tid + j * kThreads;
        kept[j] = M40Act<T>::load8(at(g < groups ? g : 0u));
    }
#pragma unroll
    for (uint32_t j = 0; j < kKeep; ++j)
#pragma unroll
        for (int i = 0; i < 8; ++i) s.take(tid + j * kThreads < groups ? M40Act<T>::to(kept[j][i]) : 0.0f);
    for (uint32_t g = tid + kKeep * kThreads; g < groups; g += kThreads) {
        const vec8 v = M40Act<T>::load8(at(g));
#pragma unroll
        for (int i = 0; i < 8; ++i) s.take(M40Act<T>::to(v[i]));
    }
    s.s2 = m40_sum64(s.s2); s.s4 = m40_sum64(s.s4); s.s6 = m40_sum64(s.s6);
    if ((tid & 63u) == 0u) { part[0][tid >> 6] = s.s2; part[1][tid >> 6] = s.s4; part[2][tid >> 6] = s.s6; }
    __syncthreads();
    s.s2 = part[0][0] + part[0][1] + part[0][2] + part[0][3];
    s.s4 = part[1][0] + part[1][1] + part[1][2] + part[1][3];
    s.s6 = part[2][0] + part[2][1] + part[2][2] + part[2][3];
    const PolyFactors f(s, act, cols, eps);
#pragma unroll
    for (uint32_t j = 0; j < kKeep; ++j) {
        const uint32_t g = tid + j * kThreads;
        if (g < groups) poly_store<T>(at(g), kept[j], g * 8u, cols, f);
    }
    for (uint32_t g = tid + kKeep * kThreads; g < groups; g += kThreads) poly_store<T>(at(g), M40Act<T>::load8(at(g)), g * 8u, cols, f);
}

// Lane l of a wave holds columns 8 (l / 16) .. of row l % 16 of each of its operand tiles, KEEP of which stay in registers.
constexpr uint32_t kTileThreads = 1024, kTileWaves = kTileThreads / 64;
template <uint32_t KEEP>
__global__ __launch_bounds__(kTileThreads) void poly_norm_tiles_kernel(m40_bf16* __restrict__ z, uint32_t ld, const float* __restrict__ act, uint32_t cols, float eps) {
    __shared__ float part[3][kTileWaves][16];
    const uint32_t lane = threadIdx.x & 63u, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), li = lane & 15u, g = lane >> 4, tiles = ld >> 5;
    m40_bf16* own = z + (size_t)blockIdx.x * tiles * kM40Tile + lane * 8u;
    m40_bf16x8 kept[KEEP];
    PolySums s;
#pragma unroll
    for (uint32_t j = 0; j < KEEP; ++j) {
        const uint32_t t = wave + j * kTileWaves;
        kept[j] = *reinterpret_cast<const m40_bf16x8*>(own + (size_t)(t < tiles ? t : 0u) * kM40Tile);
    }
#pragma unroll
    for (uint32_t j = 0; j < KEEP; ++j) {
        const float live = wave + j * kTileWaves < tiles ? 1.0f : 0.0f;
#pragma unroll
        for (int i = 0; i < 8; ++i) s.take(static_cast<float>(kept[j][i]) * live);
        asm volatile("" : "+v"(kept[j]));        // stays in bf16: its values in f32 are formed again for the result
    }
    for (uint32_t t = wave + KEEP * kTileWaves; t < tiles; t += kTileWaves) {
        const m40_bf16x8 v = *reinterpret_cast<const m40_bf16x8*>(own + (size_t)t * kM40Tile);
#pragma unroll
        for (int i = 0; i < 8; ++i) s.take(static_cast<float>(v[i]));
    }
    s.s2 = m40_add_xor32(m40_add_xor16(s.s2));
    s.s4 = m40_add_xor32(m40_add_xor16(s.s4));
    s.s6 = m40_add_xor32(m40_add_xor16(s.s6));
    if (g == 0u) { part[0][wave][li] = s.s2; part[1][wave][li] = s.s4; part[2][wave][li] = s.s6; }
    __syncthreads();
    PolySums all;
#pragma unroll
    for (uint32_t w = 0; w < kTileWaves; ++w) {
        all.s2 += part[0][w][li];
        all.s4 += part[1][w][li];
        all.s6 += part[2][w][li];
    }
    const PolyFactors f(all, act, cols, eps);
#pragma unroll
    for (uint32_t j = 0; j < KEEP; ++j) {
        const uint32_t t = wave + j * kTileWaves;
        if (t < tiles) poly_store<m40_bf16>(own + (size_t)t * kM40Tile, kept[j], t * 32u + g * 8u, cols, f);
    }
    for (uint32_t t = wave + KEEP * kTileWaves; t < tiles; t += kTileWaves)
        poly_store<m40_bf16>(own + (size_t)t * kM40Tile, *reinterpret_cast<const m40_bf16x8*>(own + (size_t)t * kM40Tile), t * 32u + g * 8u, cols, f);
}

template <class T>
void launch_split(hipStream_t stream, M40llmSpaceSplit s, bool vec) {
    // heads without padding lie side by side in the rows on both sides: as many together as fill the lanes
    auto together = [](uint32_t& heads, uint32_t& size) {
        if (size % 32u != 0) return;
        for (uint32_t n = 128u / size; n > 1u; --n)
            if (heads % n == 0) {
                heads /= n;
                size *= n;
                return;
            }
    };
    together(s.heads, s.vdim);
    together(s.kv_heads, s.dim);
    const dim3 grid((s.rows + 15u) / 16u, 2u * s.kv_heads + s.heads);
    const uint32_t most = s.dim > s.vdim ? s.dim : s.vdim;
    if (!vec) space_split_kernel<T, 1, 16><<<grid, kThreads, 0, stream>>>(s);
    else if (most <= 64u) space_split_kernel<T, 4, 1><<<grid, kThreads, 0, stream>>>(s);
    else if (most <= 128u) space_split_kernel<T, 4, 2><<<grid, kThreads, 0, stream>>>(s);
    else space_split_kernel<T, 4, 4><<<grid, kThreads, 0, stream>>>(s);
}
template <class T>
void launch_group_norm(hipStream_t stream, const GroupNormArgs& a, bool vec) {
    if (a.part <= 1024u || a.groups >= 16u) {
        const dim3 grid(a.rows, (a.groups + 3u) / 4u);
        if (vec) gate_group_norm_kernel<T, 64, true><<<grid, kThreads, 0, stream>>>(a);
        else gate_group_norm_kernel<T, 64, false><<<grid, kThreads, 0, stream>>>(a);
    } else {
        const dim3 grid(a.rows, a.groups);
        if (vec) gate_group_norm_kernel<T, 256, true><<<grid, kThreads, 0, stream>>>(a);
        else gate_group_norm_kernel<T, 256, false><<<grid, kThreads, 0, stream>>>(a);
    }
}

int launched() { return hipGetLastError() == hipSuccess ? 0 : -2; }

}  // namespace

extern "C" {

int m40llm_ext_token_mix_async(M40llmCudaContext* ctx, const M40llmTokenMix* m, uint32_t stream_kind) {
    if (!ctx || !m || !m->h || !m->mu || !m->state || !m->out || !m->portions || !m->row_pos || !m->row_back) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    if (m->act_dtype > 1u || m->rows == 0 || m->ld == 0 || m->ld % 32u != 0 || m->mixes == 0 || m->n_portions == 0) return -3;
    for (const void* p : {m->h, m->mu, static_cast<const void*>(m->state), static_cast<const void*>(m->out)})
        if (!m40_aligned16(p)) return -3;
    (void)hipGetLastError();
    if (m->act_dtype == M40LLM_ACT_F32) token_mix_kernel<float><<<m->rows + m->n_portions, kThreads, 0, stream>>>(*m);
    else token_mix_kernel<m40_bf16><<<m->rows + m->n_portions, kThreads, 0, stream>>>(*m);
    return launched();
}

int m40llm_ext_space_split_async(M40llmCudaContext* ctx, const M40llmSpaceSplit* s, uint32_t stream_kind) {
    if (!ctx || !s || !s->proj || !s->conv || !s->bias || !s->out || !s->row_slot || !s->row_pos || !s->row_back) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    const uint64_t cols = 2ull * s->kv_heads * s->dim + (uint64_t)s->heads * s->vdim;
    const uint64_t out_cols = 2ull * s->kv_heads * ((s->dim + 31u) / 32u * 32u) + (uint64_t)s->heads * ((s->vdim + 31u) / 32u * 32u);
    if (s->act_dtype > 1u || s->rows == 0 || s->heads == 0 || s->kv_heads == 0 || s->dim == 0 || s->dim > 256u || s->vdim == 0 || s->vdim > 256u || s->taps == 0 ||
        2u * s->kv_heads + s->heads > 65535u || s->ld_proj < cols || s->ld_out < out_cols || s->ld_out % 32u != 0 || !m40_aligned16(s->out))
        return -3;
    if (s->taps > 1u && (!s->conv_state || s->ld_state < cols)) return -4;
    bool vec = s->dim % 4u == 0 && s->vdim % 4u == 0 && s->ld_proj % 4u == 0 && s->ld_state % 4u == 0;
    for (const void* p : {s->proj, s->conv, s->bias, static_cast<const void*>(s->conv_state)}) vec = vec && m40_aligned16(p);
    (void)hipGetLastError();
    if (s->act_dtype == M40LLM_ACT_F32) launch_split<float>(stream, *s, vec);
    else launch_split<m40_bf16>(stream, *s, vec);
    return launched();
}

int m40llm_ext_gate_group_norm_rows_async(M40llmCudaContext* ctx, const void* d_y, uint64_t ld_y, const void* d_gate, uint64_t ld_gate, const void* d_w, uint32_t rows,
                                          uint32_t cols, uint32_t groups, float eps, void* d_out, uint32_t ld_out, uint32_t act_dtype, uint32_t stream_kind) {
    if (!ctx || !d_y || !d_gate || !d_w || !d_out) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    if (rows == 0 || cols == 0 || groups == 0 || groups > 65535u || cols % groups != 0 || ld_out < cols || ld_out % 32u != 0 || ld_y < cols || ld_gate < cols || act_dtype > 1u ||
        !m40_aligned16(d_out))
        return -3;
    const GroupNormArgs a{static_cast<const float*>(d_y), static_cast<const float*>(d_gate), static_cast<const float*>(d_w), (size_t)ld_y, (size_t)ld_gate, rows, cols, groups,
                          cols / groups, eps, d_out, ld_out};
    const bool vec = a.part % 8u == 0 && ld_y % 4u == 0 && ld_gate % 4u == 0 && m40_aligned16(d_y) && m40_aligned16(d_gate) && m40_aligned16(d_w);
    (void)hipGetLastError();
    if (act_dtype == M40LLM_ACT_F32) launch_group_norm<float>(stream, a, vec);
    else launch_group_norm<m40_bf16>(stream, a, vec);
    return launched();
}

int m40llm_ext_poly_norm_rows_async(M40llmCudaContext* ctx, void* d_z, uint32_t ld, const void* d_act, uint32_t rows, uint32_t cols, float eps, uint32_t act_dtype,
                                    uint32_t stream_kind) {
    if (!ctx || !d_z || !d_act) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    if (rows == 0 || cols == 0 || ld < cols || ld % 32u != 0 || act_dtype > 1u || !m40_aligned16(d_z)) return -3;
    const float* act = static_cast<const float*>(d_act);
    (void)hipGetLastError();
    if (act_dtype == M40LLM_ACT_F32) {
        poly_norm_rows_kernel<float><<<rows, kThreads, 0, stream>>>(static_cast<float*>(d_z), ld, act, rows, cols, eps);
    } else if (rows < 1024u) {
        poly_norm_rows_kernel<m40_bf16><<<rows, kThreads, 0, stream>>>(static_cast<m40_bf16*>(d_z), ld, act, rows, cols, eps);
    } else {
        const uint32_t grid = (rows + 15u) / 16u;
        if (ld <= 32u * 12u * kTileWaves) poly_norm_tiles_kernel<12><<<grid, kTileThreads, 0, stream>>>(static_cast<m40_bf16*>(d_z), ld, act, cols, eps);
        else poly_norm_tiles_kernel<22><<<grid, kTileThreads, 0, stream>>>(static_cast<m40_bf16*>(d_z), ld, act, cols, eps);
    }
    return launched();
}

}  // extern "C"
