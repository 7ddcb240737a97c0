// Causal convolution over time per column, as the split kernels apply it to projected rows: 16 lanes a row, lane l columns in groups of W at
// W (l + 16 i), N groups at most (W 4: every size and offset a multiple of 4).
//
// What precedes a portion's first row lies in a ring by position, entry p % (taps - 1).  The only row of a portion overwrites the oldest
// entry, which it has read, with its own.
#pragma once

#include "packed_gemm.hpp"

template <int W> struct M40Columns { float v[W]; };
template <int W>
__device__ __forceinline__ M40Columns<W> m40_load_columns(const float* p) {
    M40Columns<W> c;
    if (W == 4) {
        const float4 t = *reinterpret_cast<const float4*>(p);
        c.v[0] = t.x; c.v[W > 1 ? 1 : 0] = t.y; c.v[W > 2 ? 2 : 0] = t.z; c.v[W > 3 ? 3 : 0] = t.w;
    } else {
#pragma unroll
        for (int k = 0; k < W; ++k) c.v[k] = p[k];
    }
    return c;
}
template <class T, int W>
__device__ __forceinline__ void m40_store_columns(T* p, const float (&v)[W]) {
    if (W == 4) m40_store4<T>(p, m40_float4{v[0], v[W > 1 ? 1 : 0], v[W > 2 ? 2 : 0], v[W > 3 ? 3 : 0]});
    else {
#pragma unroll
        for (int k = 0; k < W; ++k) p[k] = M40Act<T>::from(v[k]);
    }
}

struct M40ConvRow {
    const float* u;            // the unit's first column of this row
    size_t ld;                 // from row to row
    const float* w;            // the unit's first column of the weights, [taps][all]
    uint32_t all, taps;        // taps 0: the columns as they are
    float* state;              // the unit's first column of the slot's ring
    size_t ld_state;
    uint32_t pos, info;        // info: rows of the portion before this one, bit 31 where it is the only one
};
// y[i] = the n columns of the unit behind the convolution; zero past them
template <int W, int N>
__device__ __forceinline__ void m40_short_conv(const M40ConvRow& r, uint32_t n, uint32_t lane, float (&y)[N][W]) {
    uint32_t c[N];
    bool live[N];
    M40Columns<W> now[N];
#pragma unroll
    for (int i = 0; i < N; ++i) {
        c[i] = W * (lane + 16u * i);
        live[i] = c[i] < n;
        if (!live[i]) c[i] = 0u;             // loads of columns past the unit go to its first
        now[i] = m40_load_columns<W>(r.u + c[i]);
    }
    if (r.taps) {
        const uint32_t keep = r.taps - 1u, back = r.info & 0x7fffffffu;
#pragma unroll
        for (int i = 0; i < N; ++i) {
            const M40Columns<W> wn = m40_load_columns<W>(r.w + (size_t)keep * r.all + c[i]);
#pragma unroll
            for (int k = 0; k < W; ++k) y[i][k] = wn.v[k] * now[i].v[k];
        }
#pragma unroll 4
        for (uint32_t d = 1; d <= keep; ++d) {               // rows back; loads under selected addresses, none behind a branch
            const bool here = d <= back, some = d <= r.pos;
            const float* src = here ? r.u - (size_t)d * r.ld : some ? r.state + (size_t)((r.pos - d) % keep) * r.ld_state : r.u;
            const float f = some ? 1.0f : 0.0f;
#pragma unroll
            for (int i = 0; i < N; ++i) {
                const M40Columns<W> before = m40_load_columns<W>(src + c[i]), wd = m40_load_columns<W>(r.w + (size_t)(keep - d) * r.all + c[i]);
#pragma unroll
                for (int k = 0; k < W; ++k) y[i][k] = fmaf(wd.v[k] * f, before.v[k], y[i][k]);
            }
        }
        if (r.info >> 31 && keep) {
            float* own = r.state + (size_t)(r.pos % keep) * r.ld_state;
#pragma unroll
            for (int i = 0; i < N; ++i)
                if (live[i]) m40_store_columns<float, W>(own + c[i], now[i].v);
        }
    } else {
#pragma unroll
        for (int i = 0; i < N; ++i)
#pragma unroll
            for (int k = 0; k < W; ++k) y[i][k] = now[i].v[k];
    }
#pragma unroll
    for (int i = 0; i < N; ++i)
#pragma unroll
        for (int k = 0; k < W; ++k) y[i][k] = live[i] ? y[i][k] : 0.0f;
}
template <int W, int N>
__device__ __forceinline__ float m40_sum_squares16(const float (&y)[N][W]) {      // of a row's 16 lanes
    float ss = 0.0f;
#pragma unroll
    for (int i = 0; i < N; ++i)
#pragma unroll
        for (int k = 0; k < W; ++k) ss = fmaf(y[i][k], y[i][k], ss);
    return m40_sum16(ss);
}
