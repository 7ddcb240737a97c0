// Recurrent layers with a matrix state, token after token: decoded tokens, and every portion in f32.  A workgroup holds a head's whole state
// in registers, so that the head's norm and gate follow in the same launch.
#include "memory_rules.hpp"
#include "memory_launch.hpp"

namespace {

constexpr uint32_t kThreads = 512, kWaves = kThreads / 64;

// A thread holds four value columns (VG groups of them in all, a power of two) of every (512 / VG)-th key dimension, R of them.
template <class T, int VG, int R, M40MemoryRule RULE>
__global__ __launch_bounds__(kThreads) void memory_serial_kernel(M40MemoryArgs a) {
    constexpr bool DELTA = RULE == kM40Delta, MEMORY = RULE == kM40Memory, MIXING = RULE == kM40Mixing;
    constexpr uint32_t kRows = kThreads / VG, kMost = 256;
    __shared__ m40_float4 part[2][kWaves][VG], part_q[DELTA ? 2 : 1][DELTA ? kWaves : 1][DELTA ? VG : 1];
    __shared__ float extra[2][kWaves];             // n . q, k . q, or (bonus k) . q
    __shared__ float lq[2][kMost], lk[2][kMost], lg[MEMORY ? 1 : 2][MEMORY ? 1 : kMost], lb[MIXING ? 2 : 1][MIXING ? kMost : 1];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, vg = tid % VG, d0 = tid / VG, v0 = 4u * vg;
    const uint32_t* portion = a.portions + 4 * blockIdx.x;
    const uint32_t row0 = portion[0], n = portion[1], head = blockIdx.y, shared_head = head / a.share, dim = a.dim;
    const uint32_t v_left = v0 < a.vdim ? a.vdim - v0 : 0u;
    const bool v_vec = a.vdim % 4u == 0 && a.ld % 4u == 0 && m40_aligned16(a.v), g_vec = a.vdim % 4u == 0 && a.ld_gate % 4u == 0 && m40_aligned16(a.gate);
    float* state = a.state + ((size_t)portion[2] * a.heads + head) * a.head_floats;
    float* n_state = state + (size_t)dim * a.v4;
    const bool fresh = a.row_pos[row0] == 0u;
    m40_float4 S[R];
    float nv[MEMORY ? R : 1], top = 0.0f;
#pragma unroll
    for (int i = 0; i < R; ++i) {
        const uint32_t d = d0 + kRows * i;
        S[i] = m40_float4{0.f, 0.f, 0.f, 0.f};
        if (d < dim && v0 < a.v4 && !fresh) S[i] = *reinterpret_cast<const m40_float4*>(state + (size_t)d * a.v4 + v0);
        if (MEMORY) nv[MEMORY ? i : 0] = d < dim && vg == 0u && !fresh ? n_state[d] : 0.0f;
    }
    if (MEMORY && !fresh) top = n_state[a.dim4()];
    const float rate = DELTA ? expf(a.A_log[head]) : 0.0f;
    for (uint32_t t = 0; t < n; ++t) {
        const uint32_t row = row0 + t, ph = t & 1u;
        if (tid < dim) {
            const float q = a.q[(size_t)row * a.ld + shared_head * dim + tid] * a.q_factor;
            lq[ph][tid] = q;
            if (DELTA) lg[DELTA ? ph : 0][DELTA ? tid : 0] = expf(-rate * m40_channel_step(a, row, head, tid));
            if (MIXING) {
                lg[MIXING ? ph : 0][MIXING ? tid : 0] = expf(-expf(a.a[(size_t)row * a.ld_a + head * dim + tid] + a.dt_bias[head * dim + tid]));
                lb[MIXING ? ph : 0][MIXING ? tid : 0] = q * a.bonus[head * dim + tid];
            }
        } else if (tid >= kMost && tid - kMost < dim) {
            lk[ph][tid - kMost] = a.k[(size_t)row * a.ld + shared_head * dim + tid - kMost];
        }
        const m40_float4 v = m40_load4(a.v + (size_t)row * a.ld + head * a.vdim + v0, v_left, v_vec);
        m40_float4 z = {0.f, 0.f, 0.f, 0.f}, w = z;      // gate and norm weights of the columns this thread will finish
        if (wave == 0u && lane < VG) {
            z = m40_load4(a.gate + (size_t)row * a.ld_gate + head * a.vdim + v0, v_left, g_vec);
            w = m40_load4(a.norm + head * a.norm_stride + v0, v_left, false);
        }
        float keep = 0.0f, add = 0.0f, beta = 0.0f;
        if (DELTA) {
            beta = m40_sigmoid(a.beta[(size_t)row * a.ld_beta + head]);
        } else if (MEMORY) {
            const float i = m40_log_input_gate(a, a.i[(size_t)row * a.ld + head], head), f = m40_log_forget_gate(a, a.f[(size_t)row * a.ld + head], head), next = fmaxf(f + top, i);
            keep = expf(f + top - next);
            add = expf(i - next);
            top = next;
        }
        __syncthreads();
        m40_float4 o = {0.f, 0.f, 0.f, 0.f}, s = o;
        float x = 0.0f;
#pragma unroll
        for (int i = 0; i < R; ++i) {
            const uint32_t d = d0 + kRows * i;
            if (d >= dim) continue;
            const float q = lq[ph][d], k = lk[ph][d];
            if (DELTA) {
                S[i] *= lg[DELTA ? ph : 0][DELTA ? d : 0];
                s += S[i] * k;
                if (vg == 0u) x = fmaf(k, q, x);
            } else if (MIXING) {
                if (vg == 0u) x = fmaf(lb[MIXING ? ph : 0][MIXING ? d : 0], k, x);
                o += S[i] * q;
                S[i] = S[i] * lg[MIXING ? ph : 0][MIXING ? d : 0] + v * k;
            } else {
                S[i] = S[i] * keep + v * (add * k);
                if (vg == 0u) {
                    nv[MEMORY ? i : 0] = fmaf(nv[MEMORY ? i : 0], keep, add * k);
                    x = fmaf(nv[MEMORY ? i : 0], q, x);
                }
            }
            if (!MIXING) o += S[i] * q;
        }
        // lanes of a wave that hold the same columns
        auto over_lanes = [](float y) {
            if (VG == 16) y = m40_add_xor16(y);
            if (VG <= 32) y = m40_add_xor32(y);
            return y;
        };
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            o[r] = over_lanes(o[r]);
            if (DELTA) s[r] = over_lanes(s[r]);
        }
        x = over_lanes(x);
        if (lane < VG) {
            part[ph][wave][lane] = o;
            if (DELTA) part_q[DELTA ? ph : 0][DELTA ? wave : 0][DELTA ? lane : 0] = s;
        }
        if (lane == 0u) extra[ph][wave] = x;
        __syncthreads();
        m40_float4 u = {0.f, 0.f, 0.f, 0.f};
        if (DELTA) {
            m40_float4 read = u;
#pragma unroll
            for (uint32_t j = 0; j < kWaves; ++j) read += part_q[DELTA ? ph : 0][DELTA ? j : 0][DELTA ? vg : 0];
            u = (v - read) * beta;
#pragma unroll
            for (int i = 0; i < R; ++i) {
                const uint32_t d = d0 + kRows * i;
                if (d < dim) S[i] += u * lk[ph][d];
            }
        }
        if (wave == 0u) {
            m40_float4 y = {0.f, 0.f, 0.f, 0.f};
            float e = 0.0f;
#pragma unroll
            for (uint32_t j = 0; j < kWaves; ++j) {
                if (lane < VG) y += part[ph][j][vg];
                e += extra[ph][j];
            }
            if (DELTA) y += u * e;
            else if (MIXING) y += v * e;
            else y *= 1.0f / (fmaxf(fabsf(e), expf(-top)) + 1e-6f);
            if (lane >= VG) y = m40_float4{0.f, 0.f, 0.f, 0.f};
            const float ss = m40_sum64(y[0] * y[0] + y[1] * y[1] + y[2] * y[2] + y[3] * y[3]);       // columns past vdim are zero
            const float inv = a.out_factor / sqrtf(ss / (float)a.vdim + a.eps);
#pragma unroll
            for (int r = 0; r < 4; ++r) y[r] *= inv * w[r] * (MIXING ? m40_silu(z[r]) : m40_sigmoid(z[r]));
            if (lane < VG && v_left)
                m40_store_packed<T>(static_cast<T*>(a.out), (int)row, (int)(a.out_col + head * a.vdim + v0), (long)a.ld_out, y, (int)v_left, a.vdim % 4u == 0 && a.out_col % 4u == 0);
        }
    }
#pragma unroll
    for (int i = 0; i < R; ++i) {
        const uint32_t d = d0 + kRows * i;
        if (d < dim && v0 < a.v4) *reinterpret_cast<m40_float4*>(state + (size_t)d * a.v4 + v0) = S[i];
        if (MEMORY && d < dim && vg == 0u) n_state[d] = nv[MEMORY ? i : 0];
    }
    if (MEMORY && tid == 0u) n_state[a.dim4()] = top;
}

template <class T, int VG, int R, M40MemoryRule RULE>
void go(hipStream_t stream, const M40MemoryArgs& a, uint32_t n_portions) {
    memory_serial_kernel<T, VG, R, RULE><<<dim3(n_portions, a.heads), kThreads, 0, stream>>>(a);
}
template <class T, M40MemoryRule RULE>
void pick(hipStream_t stream, const M40MemoryArgs& a, uint32_t n) {
    if (a.vdim <= 64u) {
        if (a.dim <= 64u) go<T, 16, 2, RULE>(stream, a, n);
        else if (a.dim <= 128u) go<T, 16, 4, RULE>(stream, a, n);
        else go<T, 16, 8, RULE>(stream, a, n);
    } else if (a.vdim <= 128u) {
        if (a.dim <= 64u) go<T, 32, 4, RULE>(stream, a, n);
        else if (a.dim <= 128u) go<T, 32, 8, RULE>(stream, a, n);
        else go<T, 32, 16, RULE>(stream, a, n);
    } else {
        if (a.dim <= 64u) go<T, 64, 8, RULE>(stream, a, n);
        else if (a.dim <= 128u) go<T, 64, 16, RULE>(stream, a, n);
        else go<T, 64, 32, RULE>(stream, a, n);
    }
}

template <class T>
void pick_rule(hipStream_t stream, const M40MemoryArgs& a, M40MemoryRule rule, uint32_t n) {
    if (rule == kM40Delta) pick<T, kM40Delta>(stream, a, n);
    else if (rule == kM40Mixing) pick<T, kM40Mixing>(stream, a, n);
    else pick<T, kM40Memory>(stream, a, n);
}

}  // namespace

int m40_launch_memory_serial(hipStream_t stream, const M40MemoryArgs& a, M40MemoryRule rule, uint32_t act_dtype, uint32_t n_portions) {
    if (act_dtype == M40LLM_ACT_F32) pick_rule<float>(stream, a, rule, n_portions);
    else pick_rule<m40_bf16>(stream, a, rule, n_portions);
    return hipGetLastError() == hipSuccess ? 0 : -2;
}
