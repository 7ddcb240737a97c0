// Tile-packed operands of the bf16 / f32 layer kernels, and the last steps ("epilogues") their matrix products share.
//
// Packed matrix [N][K]: 16 x 32 tiles, tile (n / 16, k / 32) at index (n / 16) * k_tiles + k / 32, 512 elements each in the
// lane order of the 16x16x32 matrix instruction: element (n, k) sits at ((k % 32) / 8 * 16 + n % 16) * 8 + k % 8.  A wave's
// 16-byte load per lane is then one contiguous kilobyte and is already the instruction's operand.  Rows and columns past
// the matrix are zero.  The pages of a latent cache use the same order with tokens as rows.
#pragma once

#include "common.hpp"

#ifdef __HIPCC__
typedef __bf16 m40_bf16;
typedef __bf16 m40_bf16x8 __attribute__((ext_vector_type(8)));
typedef __bf16 m40_bf16x4 __attribute__((ext_vector_type(4)));
typedef float m40_f32x8 __attribute__((ext_vector_type(8)));

constexpr int kM40Tile = 512;            // elements of a 16 x 32 tile

__device__ __forceinline__ size_t m40_tile_offset(uint32_t row_in_tile, uint32_t k_in_tile) {
    return (size_t)(((k_in_tile >> 3) * 16u + row_in_tile) * 8u + (k_in_tile & 7u));
}
__device__ __forceinline__ float m40_bf16_bits(uint16_t b) { return __builtin_bit_cast(float, (uint32_t)b << 16); }

template <class T> struct M40Act;
template <> struct M40Act<m40_bf16> {
    typedef m40_bf16x8 vec8;
    static __device__ __forceinline__ vec8 load8(const m40_bf16* p) { return *reinterpret_cast<const m40_bf16x8*>(p); }
    static __device__ __forceinline__ m40_bf16 from(float x) { return static_cast<m40_bf16>(x); }
    static __device__ __forceinline__ float to(m40_bf16 x) { return static_cast<float>(x); }
    // one 16x16x32 step: bf16 products, f32 sums
    static __device__ __forceinline__ m40_float4 mma(const vec8& a, const m40_bf16x8& b, const m40_float4& c) {
        return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
    }
};
template <> struct M40Act<float> {
    typedef m40_f32x8 vec8;
    static __device__ __forceinline__ vec8 load8(const float* p) {
        const float4 a = reinterpret_cast<const float4*>(p)[0], b = reinterpret_cast<const float4*>(p)[1];
        return vec8{a.x, a.y, a.z, a.w, b.x, b.y, b.z, b.w};
    }
    static __device__ __forceinline__ float from(float x) { return x; }
    static __device__ __forceinline__ float to(float x) { return x; }
    // the same step as eight f32 matrix instructions: instruction j takes element j of every lane's eight (k = 8 * (lane / 16) + j)
    static __device__ __forceinline__ m40_float4 mma(const vec8& a, const m40_bf16x8& b, m40_float4 c) {
#pragma unroll
        for (int j = 0; j < 8; ++j) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[j], static_cast<float>(b[j]), c, 0, 0, 0);
        return c;
    }
};

__device__ __forceinline__ float m40_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
// 0.5 z (1 + tanh(u)) = z / (1 + exp(-2 u)), u = sqrt(2 / pi) (z + 0.044715 z^3)
__device__ __forceinline__ float m40_gelu_tanh(float z) {
    const float u = 0.7978845608028654f * (z + 0.044715f * z * z * z);
    return z / (1.0f + expf(-2.0f * u));
}

// What happens to the sums of a product.  The instruction's result layout: lane holds rows 4 * (lane / 16) + r, column lane % 16.
// Columns count in the packed matrix (col = 16 * tile + lane % 16).
template <class T>
struct M40Epilogue {
    int kind;                      // M40LLM_PACKED_*
    int rows;                      // rows past it are not stored
    float* out_f32;                // STORE / ADD / PROJECT (its plain columns)
    T* out_act;                    // STORE_ACT / GATED / ROTATE, PROJECT (its gated columns)
    long ld_out, ld_act;           // elements from row to row
    long out_batch, act_batch;     // elements from batch (head) to batch
    int cols;                      // columns stored (STORE, ADD, STORE_ACT, GATED)
    int plain_tiles;               // PROJECT: tiles before the gate / up pairs
    const float* gate;             // GATED: logits, [rows][ld_gate], one column per batch
    long ld_gate;
    // ROTATE: columns are heads of head_width; from rot_start on they are rotated; rows below split_row put the rotated part at
    // rot_out[(row * heads + head) * ld_rot + i] instead of beside the plain part
    int head_width, rot_start, heads, split_row, rot_half;
    const float2* angles;          // [rows][rot_half] (cos, sin)
    T* rot_out;
    long ld_rot;
};

template <class T>
__device__ __forceinline__ void m40_epilogue_tile(const M40Epilogue<T>& e, int batch, int row0, int tile, int lane, const m40_float4& v) {
    const int col = tile * 16 + (lane & 15), row = row0 + 4 * (lane >> 4);
    switch (e.kind) {
        case M40LLM_PACKED_STORE:
        case M40LLM_PACKED_PROJECT:
        case M40LLM_PACKED_ADD: {
            if (e.kind != M40LLM_PACKED_PROJECT && col >= e.cols) return;
            float* o = e.out_f32 + batch * e.out_batch + (long)row * e.ld_out + col;
#pragma unroll
            for (int r = 0; r < 4; ++r)
                if (row + r < e.rows) {
                    float* p = o + r * e.ld_out;
                    *p = e.kind == M40LLM_PACKED_ADD ? *p + v[r] : v[r];
                }
            return;
        }
        case M40LLM_PACKED_STORE_ACT: {
            if (col >= e.cols) return;
            T* o = e.out_act + batch * e.act_batch + (long)row * e.ld_act + col;
#pragma unroll
            for (int r = 0; r < 4; ++r)
                if (row + r < e.rows) o[r * e.ld_act] = M40Act<T>::from(v[r]);
            return;
        }
        case M40LLM_PACKED_GATED: {
            if (col >= e.cols) return;
            T* o = e.out_act + batch * e.act_batch + (long)row * e.ld_act + col;
#pragma unroll
            for (int r = 0; r < 4; ++r)
                if (row + r < e.rows)
                    o[r * e.ld_act] = M40Act<T>::from(v[r] * m40_sigmoid(e.gate[(long)(row + r) * e.ld_gate + batch]));
            return;
        }
        case M40LLM_PACKED_ROTATE: {
            const int head = col / e.head_width, i = col - head * e.head_width;
            if (i < e.rot_start) {       // a tile lies on one side: both parts are multiples of 32 wide
                T* o = e.out_act + (long)row * e.ld_act + col;
#pragma unroll
                for (int r = 0; r < 4; ++r)
                    if (row + r < e.rows) o[r * e.ld_act] = M40Act<T>::from(v[r]);
                return;
            }
            const int j = i - e.rot_start;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const float other = m40_dpp_f<M40_DPP_XOR1>(v[r]);      // the pair's other half sits in the neighbouring lane
                if (row + r >= e.rows) continue;
                const float2 cs = e.angles[(long)(row + r) * e.rot_half + (j >> 1)];
                const float y = (j & 1) ? fmaf(v[r], cs.x, other * cs.y) : fmaf(v[r], cs.x, -(other * cs.y));
                T* o = row + r < e.split_row ? e.rot_out + ((long)(row + r) * e.heads + head) * e.ld_rot + j
                                             : e.out_act + (long)(row + r) * e.ld_act + col;
                *o = M40Act<T>::from(y);
            }
            return;
        }
    }
}
// PROJECT, columns from plain_tiles on: tiles come in pairs (gate, up); pair p gives 16 activated columns
template <class T>
__device__ __forceinline__ void m40_epilogue_pair(const M40Epilogue<T>& e, int row0, int pair, int lane, const m40_float4& g,
                                                  const m40_float4& u) {
    const int col = pair * 16 + (lane & 15), row = row0 + 4 * (lane >> 4);
    T* o = e.out_act + (long)row * e.ld_act + col;
#pragma unroll
    for (int r = 0; r < 4; ++r)
        if (row + r < e.rows) o[r * e.ld_act] = M40Act<T>::from(m40_gelu_tanh(g[r]) * u[r]);
}
#endif  // __HIPCC__
