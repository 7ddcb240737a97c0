// Residual streams: the end of one sublayer and the beginning of the next in one launch.  Every stream becomes a mixture of all old ones plus
// its share of the sublayer's output, and what the next sublayer reads is a weighted sum of the new streams, normed.
#include "packed_gemm.hpp"

namespace {

constexpr int kThreads = 256;

__device__ __forceinline__ float block_sum(float v, float* scratch) {
    v = m40_sum64(v);
    if ((threadIdx.x & 63u) == 0u) scratch[threadIdx.x >> 6] = v;
    __syncthreads();
    float s = scratch[0];
#pragma unroll
    for (int i = 1; i < kThreads / 64; ++i) s += scratch[i];
    return s;
}
template <class T, bool VEC>
__device__ __forceinline__ void load8(const T* src, uint32_t at, uint32_t width, float (&v)[8]) {
    if (VEC) {
        const typename M40Act<T>::vec8 t = M40Act<T>::load8(src + at);
#pragma unroll
        for (int i = 0; i < 8; ++i) v[i] = M40Act<T>::to(t[i]);
    } else {
#pragma unroll
        for (uint32_t i = 0; i < 8; ++i) v[i] = at + i < width ? M40Act<T>::to(src[at + i]) : 0.0f;
    }
}
template <bool VEC>
__device__ __forceinline__ void store8(float* dst, uint32_t at, uint32_t width, const float (&v)[8]) {
    if (VEC) {
        reinterpret_cast<float4*>(dst + at)[0] = make_float4(v[0], v[1], v[2], v[3]);
        reinterpret_cast<float4*>(dst + at)[1] = make_float4(v[4], v[5], v[6], v[7]);
    } else {
#pragma unroll
        for (uint32_t i = 0; i < 8; ++i)
            if (at + i < width) dst[at + i] = v[i];
    }
}

// A thread takes groups of eight neighbouring columns in all streams and keeps the sums of two of them in registers (width up to 4096);
// beyond, they are formed again from the streams it has written.  S: streams, or (above four) the most there can be.
template <class T, int S, bool VEC>
__global__ __launch_bounds__(kThreads) void stream_update_kernel(M40llmStreamUpdate a) {
    __shared__ float scratch[kThreads / 64];
    constexpr uint32_t kGroups = 2;
    const uint32_t row = a.row_index ? a.row_index[blockIdx.x] : m40_tile_row(blockIdx.x, a.rows), width = a.width, groups = (a.w ? a.ld_h : (width + 7u) & ~7u) / 8u, streams = S <= 4 ? (uint32_t)S : a.streams;
    const float *mix = static_cast<const float*>(a.mix), *share = static_cast<const float*>(a.share), *take = static_cast<const float*>(a.take);
    const float* x0 = a.x0 ? static_cast<const float*>(a.x0) + (size_t)row * width : nullptr;
    float* xs = static_cast<float*>(a.streams_x) + (size_t)row * width;
    const bool write = a.place || a.n_planes;
    // up to four streams: all coefficients in registers before anything is stored
    constexpr bool kFew = S <= 4;
    float mx[kFew ? S : 1][kFew ? S : 1], sh[kFew ? S : 1], tk[kFew ? S : 1];
    if (kFew) {
#pragma unroll
        for (int t = 0; t < S; ++t) {
            tk[kFew ? t : 0] = take ? take[t] : 1.0f;
            sh[kFew ? t : 0] = write ? a.mult * share[t] : 0.0f;
#pragma unroll
            for (int s = 0; s < S; ++s) mx[kFew ? s : 0][kFew ? t : 0] = write ? mix[s * S + t] : 0.0f;
        }
    }
    auto taken = [&](uint32_t t) __attribute__((always_inline)) { return kFew ? tk[kFew ? t : 0] : take ? take[t] : 1.0f; };
    auto old = [&](uint32_t s, uint32_t g, float (&v)[8]) __attribute__((always_inline)) {
        load8<float, VEC>(x0 ? x0 : xs + s * (size_t)a.stream_stride, g * 8u, width, v);
    };
    auto output = [&](uint32_t g, float (&y)[8]) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < 8; ++i) y[i] = 0.0f;
        if (a.place) {
            for (uint32_t j0 = 0; j0 < a.top; j0 += 4u) {                 // places, then rows of four experts at a time
                uint32_t at[4];
                float f[4], v[4][8];
#pragma unroll
                for (uint32_t j = 0; j < 4; ++j) {
                    const size_t pick = (size_t)row * a.top + (j0 + j < a.top ? j0 + j : j0);
                    at[j] = a.place[pick];
                    f[j] = j0 + j >= a.top ? 0.0f : a.weight ? static_cast<const float*>(a.weight)[pick] : 1.0f;
                }
#pragma unroll
                for (uint32_t j = 0; j < 4; ++j) load8<T, VEC>(static_cast<const T*>(a.expert_out) + (size_t)at[j] * a.ld_expert, g * 8u, width, v[j]);
#pragma unroll
                for (uint32_t j = 0; j < 4; ++j)
#pragma unroll
                    for (int i = 0; i < 8; ++i) y[i] = fmaf(f[j], v[j][i], y[i]);
            }
        } else {
            const float* plane = static_cast<const float*>(a.planes) + (size_t)row * width;
            for (uint32_t p = 0; p < a.n_planes; p += 2u) {
                float v[2][8];
                const bool both = p + 1u < a.n_planes;
                load8<float, VEC>(plane + p * (size_t)a.plane_stride, g * 8u, width, v[0]);
                if (both) load8<float, VEC>(plane + (p + 1u) * (size_t)a.plane_stride, g * 8u, width, v[1]);
#pragma unroll
                for (int i = 0; i < 8; ++i) y[i] += both ? v[0][i] + v[1][i] : v[0][i];
            }
        }
    };
    // the streams' new values are stored (unless nothing reads them any more); their weighted sum in u
    auto turn = [&](uint32_t g, float (&u)[8]) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < 8; ++i) u[i] = 0.0f;
        if (g * 8u >= width) return;
        float x[S][8], y[8];
#pragma unroll
        for (uint32_t s = 0; s < S; ++s)
            if (s < streams) old(s, g, x[s]);
        if (write) output(g, y);
#pragma unroll
        for (uint32_t t = 0; t < S; ++t) {
            if (t >= streams) continue;
            float z[8];
            if (write) {
                const float f = kFew ? sh[kFew ? t : 0] : a.mult * share[t];
#pragma unroll
                for (int i = 0; i < 8; ++i) z[i] = f * y[i];
#pragma unroll
                for (uint32_t s = 0; s < S; ++s)
                    if (s < streams) {
                        const float m = kFew ? mx[kFew ? s : 0][kFew ? t : 0] : mix[s * streams + t];
#pragma unroll
                        for (int i = 0; i < 8; ++i) z[i] = fmaf(m, x[s][i], z[i]);
                    }
                if (!a.discard) store8<VEC>(xs + t * (size_t)a.stream_stride, g * 8u, width, z);
            } else {
#pragma unroll
                for (int i = 0; i < 8; ++i) z[i] = x[t][i];
            }
            const float f = taken(t);
#pragma unroll
            for (int i = 0; i < 8; ++i) u[i] = fmaf(f, z[i], u[i]);
        }
    };
    auto again = [&](uint32_t g, float (&u)[8]) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < 8; ++i) u[i] = 0.0f;
        if (g * 8u >= width) return;
        for (uint32_t t = 0; t < streams; ++t) {
            float z[8];
            load8<float, VEC>(write || !x0 ? xs + t * (size_t)a.stream_stride : x0, g * 8u, width, z);
            const float f = take ? take[t] : 1.0f;
#pragma unroll
            for (int i = 0; i < 8; ++i) u[i] = fmaf(f, z[i], u[i]);
        }
    };
    float keep[kGroups][8], q = 0.0f;
#pragma unroll
    for (uint32_t j = 0; j < kGroups; ++j) {
        turn(threadIdx.x + j * kThreads, keep[j]);
#pragma unroll
        for (int i = 0; i < 8; ++i) q = fmaf(keep[j][i], keep[j][i], q);
    }
    for (uint32_t g = threadIdx.x + kGroups * kThreads; g < groups; g += kThreads) {
        float u[8];
        turn(g, u);
#pragma unroll
        for (int i = 0; i < 8; ++i) q = fmaf(u[i], u[i], q);
    }
    const float* w = static_cast<const float*>(a.w);
    float kept_w[kGroups][8];
#pragma unroll
    for (uint32_t j = 0; j < kGroups; ++j)
#pragma unroll
        for (uint32_t i = 0; i < 8; ++i) {
            const uint32_t c = (threadIdx.x + j * kThreads) * 8u + i;
            kept_w[j][i] = w && c < width ? w[c] : 0.0f;
        }
    const float inv = w ? 1.0f / sqrtf(block_sum(q, scratch) / (float)width + a.eps) : 1.0f;
    auto finish = [&](uint32_t g, const float (&u)[8], const float (&wg)[8]) __attribute__((always_inline)) {
        if (!w) {
            if (g * 8u < width) store8<VEC>(static_cast<float*>(a.x_out) + (size_t)row * width, g * 8u, width, u);
            return;
        }
        float v[8];
#pragma unroll
        for (uint32_t i = 0; i < 8; ++i) v[i] = u[i] * inv * wg[i];          // both zero past the width
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
        if (g < groups) finish(g, keep[j], kept_w[j]);
    }
    for (uint32_t g = threadIdx.x + kGroups * kThreads; g < groups; g += kThreads) {
        float u[8], wg[8];
        if (a.discard) turn(g, u);
        else again(g, u);
#pragma unroll
        for (uint32_t i = 0; i < 8; ++i) wg[i] = w && g * 8u + i < width ? w[g * 8u + i] : 0.0f;
        finish(g, u, wg);
    }
}

template <class T, int S>
void launch(hipStream_t stream, const M40llmStreamUpdate& a, bool vec) {
    if (vec) stream_update_kernel<T, S, true><<<a.rows, kThreads, 0, stream>>>(a);
    else stream_update_kernel<T, S, false><<<a.rows, kThreads, 0, stream>>>(a);
}
template <class T>
void launch_any(hipStream_t stream, const M40llmStreamUpdate& a, bool vec) {
    switch (a.streams) {
        case 1: return launch<T, 1>(stream, a, vec);
        case 2: return launch<T, 2>(stream, a, vec);
        case 3: return launch<T, 3>(stream, a, vec);
        case 4: return launch<T, 4>(stream, a, vec);
        default: return a.streams <= 8u ? launch<T, 8>(stream, a, vec) : launch<T, 16>(stream, a, vec);
    }
}

}  // namespace

extern "C" int m40llm_ext_stream_update_async(M40llmCudaContext* ctx, const M40llmStreamUpdate* u, uint32_t stream_kind) {
    if (!ctx || !u || (!u->x0 && !u->streams_x) || (u->w ? !u->h || !u->take : !u->x_out)) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    const bool write = u->place || u->n_planes;
    if (u->act_dtype > 1u || u->rows == 0 || u->width == 0 || u->streams == 0 || u->streams > M40LLM_MOST_STREAMS ||
        (u->w && (u->ld_h < u->width || u->ld_h % 32u != 0 || !m40_aligned16(u->h) || (u->h_rows && !m40_aligned16(u->h_rows)))))
        return -3;
    if (u->row_index && u->w) return -4;           // rows of h are those of the step
    if (write && (!u->streams_x || !u->mix || !u->share || (u->place ? !u->expert_out || u->top == 0 : !u->planes))) return -4;
    const bool vec = u->width % 8u == 0 && u->stream_stride % 4u == 0 && m40_aligned16(u->streams_x) && (!u->x0 || m40_aligned16(u->x0)) && (!u->x_out || m40_aligned16(u->x_out)) &&
                     (u->place ? u->ld_expert % 8u == 0 && m40_aligned16(u->expert_out) : u->plane_stride % 4u == 0 && (!u->n_planes || m40_aligned16(u->planes)));
    (void)hipGetLastError();
    if (u->act_dtype == M40LLM_ACT_F32) launch_any<float>(stream, *u, vec);
    else launch_any<m40_bf16>(stream, *u, vec);
    return hipGetLastError() == hipSuccess ? 0 : -2;
}
