// What the kernels of recurrent layers with a matrix state share: matrix memory with exponential gates (a running maximum keeps its
// exponents small; beside S a vector n), the delta rule with one decay per key channel, and time mixing (one decay per key channel, what a token
// writes is read by later tokens only, itself it sees through a bonus).  All of it is f32.
#pragma once

#include "packed_gemm.hpp"

enum M40MemoryRule { kM40Memory = M40LLM_RULE_MEMORY, kM40Delta = M40LLM_RULE_DELTA, kM40Mixing = M40LLM_RULE_MIXING };

struct M40MemoryArgs {
    uint32_t heads, share, dim, vdim, v4;          // share: heads that use one query / key head; v4: floats of a state row
    const float *q, *k, *v;                        // rows of ld floats, head after head
    size_t ld;
    const float *i, *f, *i_bias, *f_bias;          // matrix memory: gate logits of a row, ld apart
    float cap;
    const float *a, *beta, *A_log, *dt_bias;       // delta rule: decay logits (heads x dim, ld_a apart), write strength logits (ld_beta)
    const float* bonus;                            // time mixing: heads x dim; its decay logits are a + dt_bias
    size_t ld_a, ld_beta;
    const float *norm, *gate;                      // the head's norm weights (norm_stride from head to head), gate logits (heads x vdim)
    uint32_t norm_stride;
    size_t ld_gate;
    float q_factor, eps, out_factor;
    float* state;                                  // [slot][head][head_floats]: S [dim][v4], then (matrix memory) n [dim up to 4], m
    size_t head_floats;
    void* out;
    uint32_t ld_out, out_col;
    const uint32_t *portions, *chunk_base, *chunks, *row_pos;
    // chunks: a block of floats per chunk and head
    float* scratch;
    size_t block;
    uint32_t dp, vt;                               // key dimensions up to 64, 16-column value tiles (matrix memory: with a column for n)
    uint32_t at_k, at_p, at_u, at_decay, at_s, at_w, at_gate;      // parts of a block; the queries come first
    __host__ __device__ uint32_t dim4() const { return (dim + 3u) & ~3u; }
};

#ifdef __HIPCC__
constexpr float kM40Log2e = 1.4426950408889634f;
__device__ __forceinline__ float m40_soft_cap(float z, float cap) { return cap * tanhf(z / cap); }
// log(1 + e^z): max(z, 0) + log(1 + y) with y = e^-|z|, the logarithm by its series where 1 + y would round y off
__device__ __forceinline__ float m40_softplus(float z) {
    const float y = __builtin_amdgcn_exp2f(-fabsf(z) * kM40Log2e);
    const float series = y * fmaf(-y, fmaf(-y, fmaf(-y, 0.25f, 1.0f / 3.0f), 0.5f), 1.0f);
    return fmaxf(z, 0.0f) + (y < 0.03125f ? series : __builtin_amdgcn_logf(1.0f + y) * 0.6931471805599453f);
}
// logits of a row's gates
__device__ __forceinline__ float m40_log_input_gate(const M40MemoryArgs& a, float z, uint32_t head) { return m40_soft_cap(z + a.i_bias[head], a.cap); }
__device__ __forceinline__ float m40_log_forget_gate(const M40MemoryArgs& a, float z, uint32_t head) { return -m40_softplus(-m40_soft_cap(z + a.f_bias[head], a.cap)); }
// time mixing: log2 of a key channel's decay; what is below this is nothing in f32
__device__ __forceinline__ float m40_mixing_log2_decay(float z) { return fmaxf(-expf(z) * kM40Log2e, -160.0f); }
// minus the log of a key channel's decay, less the head's factor exp(A_log)
__device__ __forceinline__ float m40_channel_step(const M40MemoryArgs& a, uint32_t row, uint32_t head, uint32_t d) {
    return m40_softplus(a.a[(size_t)row * a.ld_a + head * a.dim + d] + a.dt_bias[head * a.dim + d]);
}
__device__ __forceinline__ m40_float4 m40_load4(const float* p, uint32_t left, bool vec) {        // the first `left` of four, then zeros
    if (vec && left >= 4u) return *reinterpret_cast<const m40_float4*>(p);
    m40_float4 v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (uint32_t r = 0; r < 4; ++r)
        if (r < left) v[r] = p[r];
    return v;
}
#endif
