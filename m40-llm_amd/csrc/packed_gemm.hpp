// Tile-packed operands of the bf16 / f32 layer kernels, and the last steps ("epilogues") their matrix products share.
//
// Packed matrix [N][K]: 16 x 32 tiles, tile (n / 16, k / 32) at index (n / 16) * k_tiles + k / 32, 512 elements each in the
// lane order of the 16x16x32 matrix instruction: element (n, k) sits at ((k % 32) / 8 * 16 + n % 16) * 8 + k % 8.  A wave's
// 16-byte load per lane is then one contiguous kilobyte and is already the instruction's operand.  Rows and columns past
// the matrix are zero.  Activations that products read lie in the same order (rows past the last one hold whatever is there).
// The pages of a latent cache use the same order with tokens as rows, so a page is an operand too.
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
// element (row, col) of a packed matrix whose row tiles hold k_tiles tiles
__device__ __forceinline__ size_t m40_packed_at(uint32_t row, uint32_t col, uint32_t k_tiles) {
    return ((size_t)(row >> 4) * k_tiles + (col >> 5)) * kM40Tile + m40_tile_offset(row & 15u, col & 31u);
}
__device__ __forceinline__ float m40_bf16_bits(uint16_t b) { return __builtin_bit_cast(float, (uint32_t)b << 16); }

template <class T> struct M40Act;
template <> struct M40Act<m40_bf16> {
    typedef m40_bf16x8 vec8;
    static __device__ __forceinline__ vec8 load8(const m40_bf16* p) { return *reinterpret_cast<const m40_bf16x8*>(p); }
    static __device__ __forceinline__ m40_bf16 from(float x) { return static_cast<m40_bf16>(x); }
    static __device__ __forceinline__ float to(m40_bf16 x) { return static_cast<float>(x); }
    // one 16x16x32 step, weights first: bf16 products, f32 sums
    static __device__ __forceinline__ m40_float4 mma(const m40_bf16x8& w, const vec8& a, const m40_float4& c) {
        return __builtin_amdgcn_mfma_f32_16x16x32_bf16(w, a, c, 0, 0, 0);
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
    static __device__ __forceinline__ m40_float4 mma(const m40_bf16x8& w, const vec8& a, m40_float4 c) {
#pragma unroll
        for (int j = 0; j < 8; ++j) c = __builtin_amdgcn_mfma_f32_16x16x4f32(static_cast<float>(w[j]), a[j], c, 0, 0, 0);
        return c;
    }
};

// s_waitcnt: at most vm vector-memory operations outstanding (63 = any number), no LDS operation
__device__ __forceinline__ constexpr int m40_vm_lgkm_wait(int vm) { return 0x0070 | (vm & 15) | ((vm >> 4) << 14); }
// wait, then meet the workgroup's other waves; unlike __syncthreads() it leaves loads into LDS in flight
template <int VM>
__device__ __forceinline__ void m40_wait_and_meet() {
    asm volatile("" ::: "memory");
    __builtin_amdgcn_sched_barrier(0);
    __builtin_amdgcn_s_waitcnt(m40_vm_lgkm_wait(VM));
    __builtin_amdgcn_s_barrier();
    __builtin_amdgcn_sched_barrier(0);
    asm volatile("" ::: "memory");
}
// Workgroup b of a launch over rows: workgroups are dealt to the eight dies in turn, and the rows of a 16-row tile go to one die so
// that its L2 puts their pieces of the tile's lines together.
__device__ __forceinline__ uint32_t m40_tile_row(uint32_t b, uint32_t rows) {
    return (b | 127u) < rows ? (b & ~127u) + (b & 7u) * 16u + ((b & 127u) >> 3) : b;
}
__device__ __forceinline__ float m40_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float m40_silu(float z) { return z / (1.0f + expf(-z)); }
// 0.5 z (1 + tanh(u)) = z / (1 + exp(-2 u)), u = sqrt(2 / pi) (z + 0.044715 z^3)
__device__ __forceinline__ float m40_gelu_tanh(float z) {
    const float u = 0.7978845608028654f * (z + 0.044715f * z * z * z);
    return z / (1.0f + expf(-2.0f * u));
}

// What happens to the sums of a product.  The weights are the instruction's first operand, so a lane holds one row of the result
// and four neighbouring columns of it: row lane % 16, columns 4 * (lane / 16) + r of the tile.  Columns count in the packed
// matrix (col = 16 * tile + ...).
template <class T>
struct M40Epilogue {
    int kind;                      // M40LLM_PACKED_*
    int rows;                      // rows past it are not stored
    float* out_f32;                // STORE / ADD / PROJECT (its plain columns)
    T* out_act;                    // STORE_ACT (rows), GATED / ROTATE / PROJECT's gated columns (packed), KEYS / VALUES
    long ld_out, ld_act;           // elements from row to row (packed: columns of the whole matrix, a multiple of 32)
    long out_batch, act_batch;     // elements (packed: columns) from batch (head, part of K) to batch
    int cols;                      // columns stored (STORE, ADD, STORE_ACT, GATED)
    bool vec_out, vec_act;         // four neighbouring columns may be stored at once
    int plain_tiles, act_col;      // PROJECT, SILU, SPLIT, TANH: tiles before those that go to out_act; the first column of out_act they take
    int activation;                // PROJECT
    float act_alpha, act_limit;
    const float* row_scale;        // PROJECT: on both sums of a row (NULL = ones)
    float out_scale, out_cap;      // CAP
    int n_tiles;                   // KEYS, VALUES
    const float* gate;             // GATED: logits, [rows][ld_gate], one column per batch
    long ld_gate;
    // ROTATE: columns are heads of head_width; from rot_start on they are rotated; rows below split_row put the rotated part at
    // rot_out[(row * heads + head) * ld_rot + i] instead of beside the plain part
    int head_width, rot_start, heads, split_row, rot_half;
    const float2* angles;          // [rows][rot_half] (cos, sin)
    T* rot_out;
    long ld_rot;
};

template <class T> __device__ __forceinline__ void m40_store4(T* p, const m40_float4& v);
template <> __device__ __forceinline__ void m40_store4<float>(float* p, const m40_float4& v) { *reinterpret_cast<m40_float4*>(p) = v; }
template <> __device__ __forceinline__ void m40_store4<m40_bf16>(m40_bf16* p, const m40_float4& v) {
    *reinterpret_cast<m40_bf16x4*>(p) = m40_bf16x4{static_cast<m40_bf16>(v[0]), static_cast<m40_bf16>(v[1]), static_cast<m40_bf16>(v[2]), static_cast<m40_bf16>(v[3])};
}
template <class T>
__device__ __forceinline__ void m40_store_cols(T* p, const m40_float4& v, int n, bool vec) {      // the first n of four columns
    if (vec && n >= 4) {
        m40_store4<T>(p, v);
    } else {
#pragma unroll
        for (int r = 0; r < 4; ++r)
            if (r < n) p[r] = M40Act<T>::from(v[r]);
    }
}

template <class T>
__device__ __forceinline__ void m40_store_packed(T* base, int row, int col, long ld, const m40_float4& v, int n, bool vec) {
    if (vec && n >= 4) {
        m40_store4<T>(base + m40_packed_at((uint32_t)row, (uint32_t)col, (uint32_t)ld >> 5), v);
    } else {
#pragma unroll
        for (int r = 0; r < 4; ++r)
            if (r < n) base[m40_packed_at((uint32_t)row, (uint32_t)(col + r), (uint32_t)ld >> 5)] = M40Act<T>::from(v[r]);
    }
}

template <class T>
__device__ __forceinline__ void m40_epilogue_tile(const M40Epilogue<T>& e, int batch, int row0, int tile, int lane, m40_float4 v) {
    const int col = tile * 16 + 4 * (lane >> 4), row = row0 + (lane & 15);
    if (row >= e.rows) return;
    switch (e.kind) {
        case M40LLM_PACKED_CAP:
#pragma unroll
            for (int r = 0; r < 4; ++r) v[r] = e.out_cap > 0.0f ? e.out_cap * tanhf(v[r] * e.out_scale / e.out_cap) : v[r] * e.out_scale;
            m40_store_cols<float>(e.out_f32 + (long)row * e.ld_out + col, v, e.cols - col, e.vec_out);
            return;
        case M40LLM_PACKED_SILU:
        case M40LLM_PACKED_SPLIT:
        case M40LLM_PACKED_TANH:
            if (tile >= e.plain_tiles) {
#pragma unroll
                for (int r = 0; r < 4; ++r) v[r] = e.kind == M40LLM_PACKED_SILU ? m40_silu(v[r]) : e.kind == M40LLM_PACKED_TANH ? tanhf(v[r]) : v[r];
                m40_store_packed<T>(e.out_act, row, e.act_col + col - e.plain_tiles * 16, e.ld_act, v, 4, true);
                return;
            }
            m40_store_cols<float>(e.out_f32 + (long)row * e.ld_out + col, v, 4, e.vec_out);
            return;
        case M40LLM_PACKED_STORE:
        case M40LLM_PACKED_PROJECT:
            m40_store_cols<float>(e.out_f32 + batch * e.out_batch + (long)row * e.ld_out + col, v, e.kind == M40LLM_PACKED_PROJECT ? 4 : e.cols - col,
                                  e.vec_out);
            return;
        case M40LLM_PACKED_ADD: {
            float* o = e.out_f32 + batch * e.out_batch + (long)row * e.ld_out + col;
            const int n = e.cols - col;
            if (e.vec_out && n >= 4) {
                *reinterpret_cast<m40_float4*>(o) += v;
            } else {
#pragma unroll
                for (int r = 0; r < 4; ++r)
                    if (r < n) o[r] += v[r];
            }
            return;
        }
        case M40LLM_PACKED_GATED:
            v *= m40_sigmoid(e.gate[(long)row * e.ld_gate + batch]);
            m40_store_packed<T>(e.out_act, row, (int)(batch * e.act_batch) + col, e.ld_act, v, e.cols - col, e.vec_act);
            return;
        case M40LLM_PACKED_STORE_ACT:
            m40_store_cols<T>(e.out_act + batch * e.act_batch + (long)row * e.ld_act + col, v, e.cols - col, e.vec_act);
            return;
        case M40LLM_PACKED_ROTATE: {
            const int head = col / e.head_width, j = col - head * e.head_width - e.rot_start;
            if (j < 0) {                 // a tile lies on one side: both parts are multiples of 32 wide
                m40_store_packed<T>(e.out_act, row, col, e.ld_act, v, 4, true);
                return;
            }
            const m40_float4 cs = *reinterpret_cast<const m40_float4*>(e.angles + (long)row * e.rot_half + (j >> 1));
            const m40_float4 y = {fmaf(v[0], cs[0], -(v[1] * cs[1])), fmaf(v[1], cs[0], v[0] * cs[1]), fmaf(v[2], cs[2], -(v[3] * cs[3])),
                                  fmaf(v[3], cs[2], v[2] * cs[3])};
            m40_store4<T>(row < e.split_row ? e.rot_out + ((long)row * e.heads + head) * e.ld_rot + j
                                            : e.out_act + m40_packed_at((uint32_t)row, (uint32_t)col, (uint32_t)e.ld_act >> 5), y);
            return;
        }
        case M40LLM_PACKED_KEYS:         // the result as an operand: row tile after row tile, k tiles of 32 columns
            m40_store4<T>(e.out_act + ((long)(row0 >> 4) * (e.n_tiles >> 1) + (tile >> 1)) * kM40Tile +
                              m40_tile_offset((uint32_t)lane & 15u, (uint32_t)((tile & 1) * 16 + 4 * (lane >> 4))), v);
            return;
    }
}
// VALUES: here the activations are the first operand and a lane holds column lane % 16, rows 4 * (lane / 16) + r.  Stored
// transposed, page after page of 64 rows: per column tile two operand tiles of [16 columns][32 rows], the rows of a tile in the
// order in which the result layout of a score product hands them to the next product: row 16 t + 4 g + r at place 8 g + 4 t + r.
__device__ __forceinline__ void m40_epilogue_values(const M40Epilogue<m40_bf16>& e, int row0, int tile, int lane, const m40_float4& v) {
    m40_bf16* o = e.out_act + ((long)(row0 >> 6) * e.n_tiles + tile) * (2 * kM40Tile) + ((row0 >> 5) & 1) * kM40Tile +
                  ((lane >> 4) * 16 + (lane & 15)) * 8 + ((row0 >> 4) & 1) * 4;
    m40_store4<m40_bf16>(o, v);
}
// PROJECT, columns from plain_tiles on: tiles come in pairs (gate, up); pair p gives 16 activated columns
template <class T>
__device__ __forceinline__ void m40_epilogue_pair(const M40Epilogue<T>& e, int row0, int pair, int lane, const m40_float4& g,
                                                  const m40_float4& u) {
    const int col = pair * 16 + 4 * (lane >> 4), row = row0 + (lane & 15);
    if (row >= e.rows) return;
    m40_float4 y;
    const float f = e.row_scale ? e.row_scale[row] : 1.0f;
    if (e.activation == M40LLM_LIMITED_GATE) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const float z = fminf(g[r] * f, e.act_limit), up = fminf(fmaxf(u[r] * f, -e.act_limit), e.act_limit);
            y[r] = z * m40_sigmoid(e.act_alpha * z) * (up + 1.0f);
        }
    } else {
#pragma unroll
        for (int r = 0; r < 4; ++r) y[r] = (e.activation == M40LLM_SILU ? m40_silu(g[r] * f) : m40_gelu_tanh(g[r] * f)) * (u[r] * f);
    }
    m40_store_packed<T>(e.out_act, row, e.act_col + col, e.ld_act, y, 4, true);
}
#endif  // __HIPCC__
