// Recurrent layers with a matrix state, many tokens at once, all in f32 matrix instructions.  A portion is cut at the step's rows that are
// multiples of 64; within a chunk of up to 64 tokens the recurrence is written out:
//
//   S_t = decay_t S_0 + sum_{j <= t} (k_j, decayed from j to t) u_j^T
//   o_t = (q_t, decayed from the chunk's start)^T S_0 + sum_{j <= t} P[t, j] u_j      P[t, j] = q_t . (k_j, decayed from j to t)
//
// Matrix memory: u is the values with a column of ones, whose sums are n; decays are exp of sums of log gates less the running maximum, so no
// exponent is above zero.  Delta rule: u_t = beta_t (v_t - read_t) depends on the u before it; with A[t, j] = beta_t k_t . (k_j, decayed), j < t,
// (I + A) u = beta (v - (k, decayed from the start)^T S_0), a triangular system whose solution is U_0 - W S_0.  Time mixing: u is the values;
// queries are decayed to the token before, P[t, t] is q_t . (bonus k_t).
//
// memory_scan_kernel      matrix memory: sums of log gates, the running maximum
// memory_prepare_kernel   matrix memory: P, decayed queries and keys of all chunks
// delta_prepare_kernel    delta rule: the same, and the solution of the triangular system.  Decays between two tokens are never formed as
//                         a quotient: tokens of 16-row blocks meet as a product of the row's decay since its block began and the other's to the
//                         end of its block (both at most one), tokens of one block pairwise.
// mixing_prepare_kernel   time mixing: P, decayed queries and keys, with decays as in the delta rule
// memory_walk_kernel      chunk after chunk: a workgroup holds 16 value columns of a head's state, leaves them as they are before each chunk
// memory_outputs_kernel   all chunks at once: outputs, the head's norm, the gate
//
// Operands: lane l = 16 g + i of a 16x16x4 f32 instruction holds element (i, g) of either operand and elements (4 g + r, i) of the sums.  Four
// instructions take k = 4 g + r in turn, so a lane's operands are four neighbouring floats of row i, and a tile of sums is, as it lies, the
// second operand of four more.  Everything goes through memory in "tile order" [tile][lane][4], tiles of 16 x 16, so that a wave's load is a
// contiguous kilobyte and already an operand.
#include "memory_launch.hpp"

namespace {

constexpr int kChunk = 64;
constexpr float kNever = -1e30f;

struct Chunk {
    uint32_t row0, n, slot;
    __device__ Chunk(const M40MemoryArgs& a, uint32_t c) {
        const uint32_t *portion = a.portions + 4 * a.chunks[2 * c], base = a.chunks[2 * c + 1], end = portion[0] + portion[1];
        row0 = base > portion[0] ? base : portion[0];
        n = (base + kChunk < end ? base + kChunk : end) - row0;
        slot = portion[2];
    }
};
__device__ __forceinline__ float* block_of(const M40MemoryArgs& a, uint32_t chunk, uint32_t head) { return a.scratch + ((size_t)chunk * a.heads + head) * a.block; }
__device__ __forceinline__ m40_float4 mma4(const m40_float4& x, const m40_float4& y, m40_float4 c) {
#pragma unroll
    for (int r = 0; r < 4; ++r) c = __builtin_amdgcn_mfma_f32_16x16x4f32(x[r], y[r], c, 0, 0, 0);
    return c;
}
__device__ __forceinline__ m40_float4 at4(const float* p) { return *reinterpret_cast<const m40_float4*>(p); }
__device__ __forceinline__ void put4(float* p, const m40_float4& v) { *reinterpret_cast<m40_float4*>(p) = v; }

// four columns from d on (a multiple of 4) of row t of a matrix in tile order whose rows have `tiles` tiles
__device__ __forceinline__ size_t tile_at(uint32_t t, uint32_t d, uint32_t tiles) { return (((t >> 4) * tiles + (d >> 4)) * 64u + (d >> 2 & 3u) * 16u + (t & 15u)) * 4u; }

// Dimensions d .. d + 3 of a row, zero from dim on: loads under clamped addresses, none behind a branch.  VEC: everything a multiple of 4.
template <bool VEC>
__device__ __forceinline__ m40_float4 dims4(const float* row, uint32_t d, uint32_t dim) {
    m40_float4 v;
    if (VEC) {
        v = at4(row + (d < dim ? d : 0u));
    } else {
#pragma unroll
        for (uint32_t r = 0; r < 4; ++r) v[r] = row[d + r < dim ? d + r : 0u];
    }
#pragma unroll
    for (uint32_t r = 0; r < 4; ++r) v[r] = d + r < dim ? v[r] : 0.0f;
    return v;
}

// ---- matrix memory: gates.  Part `at_gate` of a block: sums of log forget gates to t [64], log input gates [64], running maxima [64], the maximum
// before the chunk.
__global__ __launch_bounds__(1024) void memory_scan_kernel(M40MemoryArgs a) {
    __shared__ float total[2][16], best[2][16];
    const uint32_t lane = threadIdx.x & 63u, wave = threadIdx.x >> 6;
    const uint32_t *portion = a.portions + 4 * blockIdx.x, head = blockIdx.y, row0 = portion[0], end = row0 + portion[1];
    const uint32_t first = row0 / kChunk, chunks = (end - 1u) / kChunk - first + 1u, chunk0 = a.chunk_base[blockIdx.x];
    float* m_state = a.state + ((size_t)portion[2] * a.heads + head) * a.head_floats + (size_t)a.dim * a.v4 + a.dim4();
    float top = a.row_pos[row0] == 0u ? 0.0f : *m_state;
    // row of this lane in chunk c, and whether there is one
    auto row_of = [&](uint32_t c, bool& in) __attribute__((always_inline)) {
        const uint32_t base = (first + c) * kChunk, row = (base > row0 ? base : row0) + lane;
        in = c < chunks && row < end && row < base + kChunk;
        return in ? row : row0;
    };
    bool in;
    uint32_t row = row_of(wave, in), ph = 0;
    float zi = a.i[(size_t)row * a.ld + head], zf = a.f[(size_t)row * a.ld + head];          // a round ahead
    for (uint32_t c0 = 0; c0 < chunks; c0 += 16u, ph ^= 1u) {
        const uint32_t c = c0 + wave;
        const bool live = c < chunks;
        const float i = in ? m40_log_input_gate(a, zi, head) : kNever;
        float sum = in ? m40_log_forget_gate(a, zf, head) : 0.0f, most = i;       // most: the largest log input gate, decayed to this token
#pragma unroll
        for (int d = 1; d < 64; d *= 2) {
            const float s = __shfl_up(sum, d), m = __shfl_up(most, d);
            if ((int)lane >= d) {
                most = fmaxf(most, m + sum);
                sum += s;
            }
        }
        if (lane == 63u) { total[ph][wave] = sum; best[ph][wave] = most; }
        row = row_of(c + 16u, in);
        zi = a.i[(size_t)row * a.ld + head];
        zf = a.f[(size_t)row * a.ld + head];
        __syncthreads();
        float before = top;
#pragma unroll
        for (uint32_t w = 0; w < 16u; ++w) {
            if (w == wave) before = top;
            if (c0 + w < chunks) top = fmaxf(total[ph][w] + top, best[ph][w]);
        }
        if (live) {
            float* gate = block_of(a, chunk0 + c, head) + a.at_gate;
            gate[lane] = sum;
            gate[64 + lane] = i;
            gate[128 + lane] = fmaxf(sum + before, most);
            if (lane == 0u) gate[192] = before;
        }
    }
    if (threadIdx.x == 0u) *m_state = top;
}

// queries decayed from the start (tokens x key dimensions), keys decayed to the end (key dimensions x tokens), P (tokens x tokens), values (tokens x
// columns), what is left of S_0 per key dimension
template <bool VEC>
__global__ __launch_bounds__(256) void memory_prepare_kernel(M40MemoryArgs a) {
    __shared__ float sum[kChunk], input[kChunk], top[kChunk];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), g = lane >> 4, li = lane & 15;
    const Chunk c(a, blockIdx.x);
    const uint32_t head = blockIdx.y, dim = a.dim, n = c.n;
    float* out = block_of(a, blockIdx.x, head);
    const float* gate = out + a.at_gate;
    if (threadIdx.x < kChunk) {
        sum[threadIdx.x] = gate[threadIdx.x];
        input[threadIdx.x] = gate[64 + threadIdx.x];
        top[threadIdx.x] = gate[128 + threadIdx.x];
    }
    __syncthreads();
    const float m0 = gate[192], f_end = sum[n - 1u], m_end = top[n - 1u];
    auto row_of = [&](uint32_t t) { return (size_t)(c.row0 + (t < n ? t : n - 1u)) * a.ld; };
    const float *qh = a.q + (head / a.share) * dim, *kh = a.k + (head / a.share) * dim;
    // scores of this wave's 16 rows with the keys of blocks 0 .. wave
    m40_float4 s[4];
#pragma unroll
    for (int b = 0; b < 4; ++b) s[b] = m40_float4{0.f, 0.f, 0.f, 0.f};
    const uint32_t t = wave * 16 + li;
    struct Operands { m40_float4 q, k[4]; } even, odd;             // requested a step ahead
    const float *q_row = qh + row_of(t), *k_row[4] = {kh + row_of(li), kh + row_of(16 + li), kh + row_of(32 + li), kh + row_of(48 + li)};
    auto load = [&](Operands& f, uint32_t d) __attribute__((always_inline)) {
        f.q = dims4<VEC>(q_row, d + 4u * g, dim);
#pragma unroll
        for (int b = 0; b < 4; ++b) f.k[b] = dims4<VEC>(k_row[b <= wave ? b : 0], d + 4u * g, dim);
    };
    auto add = [&](const Operands& f) __attribute__((always_inline)) {
#pragma unroll
        for (int b = 0; b < 4; ++b)
            if (b <= wave) s[b] = mma4(f.k[b], f.q, s[b]);
    };
    load(even, 0u);
    for (uint32_t d = 0; d < dim; d += 32u) {
        load(odd, d + 16u);
        __builtin_amdgcn_sched_barrier(0);
        add(even);
        load(even, d + 32u);
        __builtin_amdgcn_sched_barrier(0);
        add(odd);
    }
#pragma unroll
    for (int b = 0; b < 4; ++b) {
        if (b > wave) continue;
        m40_float4 p;
#pragma unroll
        for (uint32_t r = 0; r < 4; ++r) {
            const uint32_t j = b * 16 + 4 * g + r;
            p[r] = j <= t && t < n ? s[b][r] * a.q_factor * __builtin_amdgcn_exp2f((sum[t] - sum[j] + input[j] - top[t]) * kM40Log2e) : 0.0f;
        }
        put4(out + a.at_p + ((wave * 4 + b) * 64 + lane) * 4, p);
    }
    for (uint32_t x = wave; x < a.dp / 4u; x += 4u) {            // 16 x 16 tiles: 4 dp / 16 of them
        const uint32_t tt = x / (a.dp / 16u) * 16u + li, d = x % (a.dp / 16u) * 16u + 4u * g;
        const float f = tt < n ? a.q_factor * __builtin_amdgcn_exp2f((sum[tt] + m0 - top[tt]) * kM40Log2e) : 0.0f;
        put4(out + (x * 64 + lane) * 4, dims4<VEC>(qh + row_of(tt), d, dim) * f);
    }
    for (uint32_t x = wave; x < a.dp / 16u * 4u; x += 4u) {
        const uint32_t d = x / 4u * 16u + li;
        m40_float4 y;
#pragma unroll
        for (uint32_t r = 0; r < 4; ++r) {
            const uint32_t tt = x % 4u * 16u + 4u * g + r;
            const float v = kh[row_of(tt) + (d < dim ? d : 0u)];
            y[r] = tt < n && d < dim ? v * __builtin_amdgcn_exp2f((f_end - sum[tt] + input[tt] - m_end) * kM40Log2e) : 0.0f;
        }
        put4(out + a.at_k + (x * 64 + lane) * 4, y);
    }
    for (uint32_t x = wave; x < a.vt * 4u; x += 4u) {
        const uint32_t v = x % a.vt * 16u + li;
        m40_float4 y;
#pragma unroll
        for (uint32_t r = 0; r < 4; ++r) {
            const uint32_t tt = x / a.vt * 16u + 4u * g + r;
            const float u = a.v[row_of(tt) + head * a.vdim + (v < a.vdim ? v : 0u)];
            y[r] = tt >= n || v > a.vdim ? 0.0f : v == a.vdim ? 1.0f : u;
        }
        put4(out + a.at_u + (x * 64 + lane) * 4, y);
    }
    if (threadIdx.x < a.dp) out[a.at_decay + threadIdx.x] = __builtin_amdgcn_exp2f((f_end + m0 - m_end) * kM40Log2e);
}

// loads and arithmetic stay on their side
__device__ __forceinline__ void stay() {
    asm volatile("" ::: "memory");
    __builtin_amdgcn_sched_barrier(0);
}

// ---- delta rule -------------------------------------------------------------------------------------------------------------------------
constexpr int kSlab = 32, kLdSlab = 36, kLdA = 68;
struct DeltaLds {
    float k[kChunk][kLdSlab], q[kChunk][kLdSlab], l[kChunk][kLdSlab];          // l: log2 of the decay since the 16-row block began
    float ke[kChunk][kLdSlab], qe[kChunk][kLdSlab], ks[kChunk][kLdSlab];       // k, q decayed since the block began; k decayed to its end
    float whole[4][kSlab], start[4][kSlab], rest[4][kSlab];                    // of a block: its own decay, all before it, all behind it
    float a[kChunk][kLdA];                                                     // minus A
    float inverse[4][16][20];                                                  // of I + A's diagonal blocks
    float beta[kChunk];
};
template <bool VEC>
__global__ __launch_bounds__(256, 2) void delta_prepare_kernel(M40MemoryArgs a) {
    extern __shared__ __align__(16) uint8_t delta_lds[];
    DeltaLds& lds = *reinterpret_cast<DeltaLds*>(delta_lds);
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), g = lane >> 4, li = lane & 15;
    const Chunk c(a, blockIdx.x);
    const uint32_t head = blockIdx.y, dim = a.dim, n = c.n;
    float* out = block_of(a, blockIdx.x, head);
    float* W = out + a.at_w;
    auto row_of = [&](uint32_t t) { return c.row0 + (t < n ? t : n - 1u); };
    if (tid < kChunk) lds.beta[tid] = tid < (int)n ? m40_sigmoid(a.beta[(size_t)row_of(tid) * a.ld_beta + head]) : 0.0f;
    const float rate = -kM40Log2e * expf(a.A_log[head]);
    float own_a[16], own_p[16];                     // rows of this wave's block with row lane / 4 of it, a quarter of the key dimensions
#pragma unroll
    for (int t = 0; t < 16; ++t) own_a[t] = own_p[t] = 0.0f;
    // rows of a block with those of one before it: six pairs of blocks, waves 0 and 1 for A, waves 2 and 3 for P
    const int x_of[6] = {1, 2, 2, 3, 3, 3}, y_of[6] = {0, 0, 1, 0, 1, 2};
    const bool for_p = wave >= 2;
    const int pair0 = (wave & 1) * 3;
    m40_float4 off[3];
#pragma unroll
    for (int i = 0; i < 3; ++i) off[i] = m40_float4{0.f, 0.f, 0.f, 0.f};
    const int t_in = tid >> 2, d_in = (tid & 3) * 8;
    // a slab's rows, requested a slab ahead
    struct Rows { m40_float4 k[2], q[2], z[2], bias[2]; } in;
    const bool live = t_in < (int)n;
    const size_t row_in = row_of(t_in);
    const float *k_row = a.k + row_in * a.ld + (head / a.share) * dim, *q_row = a.q + row_in * a.ld + (head / a.share) * dim, *z_row = a.a + row_in * a.ld_a + head * dim,
                *bias_row = a.dt_bias + head * dim;
    auto load = [&](uint32_t slab) __attribute__((always_inline)) {
#pragma unroll
        for (int h = 0; h < 2; ++h) {
            const uint32_t d = slab + d_in + 4 * h;
            in.k[h] = dims4<VEC>(k_row, d, dim);
            in.q[h] = dims4<VEC>(q_row, d, dim);
            in.z[h] = dims4<VEC>(z_row, d, dim);
            in.bias[h] = dims4<VEC>(bias_row, d, dim);
        }
    };
    load(0u);
    for (uint32_t slab = 0; slab < a.dp; slab += kSlab) {
#pragma unroll
        for (int h = 0; h < 2; ++h) {
            const uint32_t d = slab + d_in + 4 * h;
            m40_float4 l;
#pragma unroll
            for (uint32_t r = 0; r < 4; ++r) l[r] = live && d + r < dim ? rate * m40_softplus(in.z[h][r] + in.bias[h][r]) : 0.0f;
            put4(&lds.k[t_in][d_in + 4 * h], in.k[h] * (live ? 1.0f : 0.0f));
            put4(&lds.q[t_in][d_in + 4 * h], in.q[h] * (live ? a.q_factor : 0.0f));
            put4(&lds.l[t_in][d_in + 4 * h], l);
        }
        load(slab + kSlab);
        __syncthreads();
        if (tid < 4 * kSlab) {
            const int b = tid / kSlab, d = tid % kSlab;
            float s = 0.0f;
#pragma unroll
            for (int t = 0; t < 16; ++t) {
                s += lds.l[b * 16 + t][d];
                lds.l[b * 16 + t][d] = s;
            }
            lds.whole[b][d] = s;
        }
        __syncthreads();
        if (tid < 4 * kSlab) {
            const int b = tid / kSlab, d = tid % kSlab;
            float before = 0.0f, behind = 0.0f;
            for (int x = 0; x < 4; ++x) {
                if (x < b) before += lds.whole[x][d];
                if (x > b) behind += lds.whole[x][d];
            }
            lds.start[b][d] = __builtin_amdgcn_exp2f(before);
            lds.rest[b][d] = __builtin_amdgcn_exp2f(behind);
            if (b == 3) out[a.at_decay + slab + d] = __builtin_amdgcn_exp2f(before + lds.whole[3][d]);
        }
        {
            const int b = t_in >> 4;
#pragma unroll
            for (int h = 0; h < 2; ++h) {
                const int d = d_in + 4 * h;
                const m40_float4 l = at4(&lds.l[t_in][d]), kk = at4(&lds.k[t_in][d]), qq = at4(&lds.q[t_in][d]), end = at4(&lds.whole[b][d]);
                m40_float4 since, until;
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    since[r] = __builtin_amdgcn_exp2f(l[r]);
                    until[r] = __builtin_amdgcn_exp2f(end[r] - l[r]);
                }
                put4(&lds.ke[t_in][d], kk * since);
                put4(&lds.qe[t_in][d], qq * since);
                put4(&lds.ks[t_in][d], kk * until);
            }
        }
        __syncthreads();
        {                                           // decayed from the start, to the end
            const int b = t_in >> 4;
            const float beta = lds.beta[t_in];
#pragma unroll
            for (int h = 0; h < 2; ++h) {
                const int d = d_in + 4 * h;
                const m40_float4 f = at4(&lds.start[b][d]);
                const size_t at = tile_at(t_in, slab + d, a.dp / 16u);
                put4(out + at, at4(&lds.qe[t_in][d]) * f);
                put4(W + at, at4(&lds.ke[t_in][d]) * f * beta);
            }
#pragma unroll
            for (int h = 0; h < 2; ++h) {           // block `wave` of tokens, 16 dimensions
                const int d = h * 16 + li;
                m40_float4 y;
#pragma unroll
                for (int r = 0; r < 4; ++r) y[r] = lds.ks[wave * 16 + 4 * g + r][d] * lds.rest[wave][d];
                put4(out + a.at_k + (((slab / 16u + h) * 4u + wave) * 64 + lane) * 4, y);
            }
        }
        {                                           // pairs of the block's own rows
            const int j = lane >> 2, d = (lane & 3) * 8;
            float kj[8], lj[8];
#pragma unroll
            for (int h = 0; h < 2; ++h) {
                const m40_float4 x = at4(&lds.k[wave * 16 + j][d + 4 * h]), y = at4(&lds.l[wave * 16 + j][d + 4 * h]);
#pragma unroll
                for (int r = 0; r < 4; ++r) { kj[4 * h + r] = x[r]; lj[4 * h + r] = y[r]; }
            }
#pragma unroll
            for (int t = 0; t < 16; ++t) {
#pragma unroll
                for (int h = 0; h < 2; ++h) {
                    const m40_float4 kt = at4(&lds.k[wave * 16 + t][d + 4 * h]), qt = at4(&lds.q[wave * 16 + t][d + 4 * h]), lt = at4(&lds.l[wave * 16 + t][d + 4 * h]);
#pragma unroll
                    for (int r = 0; r < 4; ++r) {
                        const float e = kj[4 * h + r] * __builtin_amdgcn_exp2f(fminf(lt[r] - lj[4 * h + r], 0.0f));
                        own_a[t] = fmaf(kt[r], e, own_a[t]);
                        own_p[t] = fmaf(qt[r], e, own_p[t]);
                    }
                }
                if (t & 1) stay();                  // operands of two rows at a time in registers
            }
        }
        const float(*own)[kLdSlab] = for_p ? lds.qe : lds.ke;
#pragma unroll
        for (int i = 0; i < 3; ++i) {
            const int x = pair0 ? x_of[3 + i] : x_of[i], y = pair0 ? y_of[3 + i] : y_of[i];
#pragma unroll
            for (int h = 0; h < 2; ++h) {
                const int d = h * 16 + 4 * g;
                // decays of the blocks between: at most the second and the third
                const float f1 = y < 1 && x > 1 ? 1.0f : 0.0f, f2 = y < 2 && x > 2 ? 1.0f : 0.0f;
                m40_float4 f = at4(&lds.whole[1][d]) * f1 + at4(&lds.whole[2][d]) * f2;
#pragma unroll
                for (int r = 0; r < 4; ++r) f[r] = __builtin_amdgcn_exp2f(f[r]);
                off[i] = mma4(at4(&lds.ks[y * 16 + li][d]), at4(&own[x * 16 + li][d]) * f, off[i]);
            }
        }
        __syncthreads();
    }
    {
        const int j = lane >> 2;
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            float x = own_a[t], y = own_p[t];
            x += m40_dpp_f<M40_DPP_XOR1>(x);
            y += m40_dpp_f<M40_DPP_XOR1>(y);
            x += m40_dpp_f<M40_DPP_XOR2>(x);
            y += m40_dpp_f<M40_DPP_XOR2>(y);
            if ((lane & 3) == (t & 3)) {
                lds.a[wave * 16 + t][wave * 16 + j] = j < t ? -lds.beta[wave * 16 + t] * x : 0.0f;
                out[a.at_p + tile_at(wave * 16 + t, wave * 16 + (j & 12), 4u) + (j & 3)] = j <= t ? y : 0.0f;
            }
        }
#pragma unroll
        for (int i = 0; i < 3; ++i) {
            const int x = pair0 ? x_of[3 + i] : x_of[i], y = pair0 ? y_of[3 + i] : y_of[i], t = x * 16 + li;
            if (for_p) put4(out + a.at_p + ((x * 4 + y) * 64 + lane) * 4, off[i]);
            else put4(&lds.a[t][y * 16 + 4 * g], off[i] * -lds.beta[t]);
        }
    }
    __syncthreads();
    {                                               // column li of the inverse of I + A's block, by substitution
        float x[16];
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            x[t] = t == li ? 1.0f : 0.0f;
#pragma unroll
            for (int j = 0; j < t; ++j) x[t] = fmaf(lds.a[wave * 16 + t][wave * 16 + j], x[j], x[t]);
            if (t & 1) stay();
        }
        if (g == 0) {
#pragma unroll
            for (int t = 0; t < 16; ++t) lds.inverse[wave][t][li] = x[t];
        }
    }
    __syncthreads();
    const uint32_t w_tiles = a.dp / 16u;
    for (uint32_t x = wave; x < w_tiles + a.vt; x += 4u) {
        m40_float4 X[4];
#pragma unroll
        for (int b = 0; b < 4; ++b) {
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const uint32_t t = b * 16 + 4 * g + r;
                if (x < w_tiles) {
                    X[b][r] = W[tile_at(t, x * 16u + (li & 12), w_tiles) + (li & 3)];
                } else {
                    const uint32_t v = (x - w_tiles) * 16u + li;
                    const float y = a.v[(size_t)row_of(t) * a.ld + head * a.vdim + (v < a.vdim ? v : 0u)];
                    X[b][r] = v < a.vdim && t < n ? y * lds.beta[t] : 0.0f;
                }
            }
        }
#pragma unroll
        for (int b = 0; b < 4; ++b) {
#pragma unroll
            for (int j = 0; j < b; ++j) X[b] = mma4(at4(&lds.a[b * 16 + li][j * 16 + 4 * g]), X[j], X[b]);
            X[b] = mma4(at4(&lds.inverse[b][li][4 * g]), X[b], m40_float4{0.f, 0.f, 0.f, 0.f});
        }
#pragma unroll
        for (int b = 0; b < 4; ++b) {
            if (x < w_tiles) {
#pragma unroll
                for (int r = 0; r < 4; ++r) W[tile_at(b * 16 + 4 * g + r, x * 16u + (li & 12), w_tiles) + (li & 3)] = X[b][r];
            } else {
                put4(out + a.at_u + ((b * a.vt + x - w_tiles) * 64 + lane) * 4, X[b]);
            }
        }
    }
}

// ---- time mixing ------------------------------------------------------------------------------------------------------------------------
struct MixingLds {
    float k[kChunk][kLdSlab], q[kChunk][kLdSlab], l[kChunk][kLdSlab];          // l: log2 of the decay since the 16-row block began
    float qe[kChunk][kLdSlab], ks[kChunk][kLdSlab];                            // q decayed since the block began, up to the token before; k decayed to its end
    float whole[4][kSlab], start[4][kSlab], rest[4][kSlab];                    // of a block: its own decay, all before it, all behind it
};
template <bool VEC>
__global__ __launch_bounds__(256, 2) void mixing_prepare_kernel(M40MemoryArgs a) {
    __shared__ __align__(16) MixingLds lds;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), g = lane >> 4, li = lane & 15;
    const Chunk c(a, blockIdx.x);
    const uint32_t head = blockIdx.y, dim = a.dim, n = c.n;
    float* out = block_of(a, blockIdx.x, head);
    auto row_of = [&](uint32_t t) { return c.row0 + (t < n ? t : n - 1u); };
    float own[16], bonus = 0.0f;                    // own: rows of this wave's block with row lane / 4 of it, a quarter of the key dimensions
#pragma unroll
    for (int t = 0; t < 16; ++t) own[t] = 0.0f;
    // rows of a block x with those of one before it, y: six pairs, a wave's own and one of the last two
    m40_float4 off[2];
    int x_of[2], y_of[2];
#pragma unroll
    for (int i = 0; i < 2; ++i) {
        const int pair = wave + 4 * i < 6 ? wave + 4 * i : 5;
        x_of[i] = pair == 0 ? 1 : pair < 3 ? 2 : 3;
        y_of[i] = pair - x_of[i] * (x_of[i] - 1) / 2;
        off[i] = m40_float4{0.f, 0.f, 0.f, 0.f};
    }
    const int t_in = tid >> 2, d_in = (tid & 3) * 8;
    struct Rows { m40_float4 k[2], q[2], z[2], bias[2], u[2]; } in;            // a slab's rows, requested a slab ahead
    const bool live = t_in < (int)n;
    const size_t row_in = row_of(t_in);
    const float *k_row = a.k + row_in * a.ld + head * dim, *q_row = a.q + row_in * a.ld + head * dim, *z_row = a.a + row_in * a.ld_a + head * dim, *bias_row = a.dt_bias + head * dim,
                *u_row = a.bonus + head * dim;
    auto load = [&](uint32_t slab) __attribute__((always_inline)) {
#pragma unroll
        for (int h = 0; h < 2; ++h) {
            const uint32_t d = slab + d_in + 4 * h;
            in.k[h] = dims4<VEC>(k_row, d, dim);
            in.q[h] = dims4<VEC>(q_row, d, dim);
            in.z[h] = dims4<VEC>(z_row, d, dim);
            in.bias[h] = dims4<VEC>(bias_row, d, dim);
            in.u[h] = dims4<VEC>(u_row, d, dim);
        }
    };
    load(0u);
    for (uint32_t slab = 0; slab < a.dp; slab += kSlab) {
#pragma unroll
        for (int h = 0; h < 2; ++h) {
            const uint32_t d = slab + d_in + 4 * h;
            const m40_float4 k = in.k[h] * (live ? 1.0f : 0.0f), q = in.q[h] * (live ? a.q_factor : 0.0f);
            m40_float4 l;
#pragma unroll
            for (uint32_t r = 0; r < 4; ++r) {
                l[r] = live && d + r < dim ? m40_mixing_log2_decay(in.z[h][r] + in.bias[h][r]) : 0.0f;
                bonus = fmaf(q[r] * in.u[h][r], k[r], bonus);
            }
            put4(&lds.k[t_in][d_in + 4 * h], k);
            put4(&lds.q[t_in][d_in + 4 * h], q);
            put4(&lds.l[t_in][d_in + 4 * h], l);
        }
        load(slab + kSlab);
        __syncthreads();
        if (tid < 4 * kSlab) {
            const int b = tid / kSlab, d = tid % kSlab;
            float s = 0.0f;
#pragma unroll
            for (int t = 0; t < 16; ++t) {
                s += lds.l[b * 16 + t][d];
                lds.l[b * 16 + t][d] = s;
            }
            lds.whole[b][d] = s;
        }
        __syncthreads();
        if (tid < 4 * kSlab) {
            const int b = tid / kSlab, d = tid % kSlab;
            float before = 0.0f, behind = 0.0f;
            for (int x = 0; x < 4; ++x) {
                if (x < b) before += lds.whole[x][d];
                if (x > b) behind += lds.whole[x][d];
            }
            lds.start[b][d] = __builtin_amdgcn_exp2f(before);
            lds.rest[b][d] = __builtin_amdgcn_exp2f(behind);
            if (b == 3) out[a.at_decay + slab + d] = __builtin_amdgcn_exp2f(before + lds.whole[3][d]);
        }
        {
            const int b = t_in >> 4, before = t_in & 15 ? t_in - 1 : t_in;
            const float f = t_in & 15 ? 1.0f : 0.0f;
#pragma unroll
            for (int h = 0; h < 2; ++h) {
                const int d = d_in + 4 * h;
                const m40_float4 l = at4(&lds.l[t_in][d]), past = at4(&lds.l[before][d]), end = at4(&lds.whole[b][d]);
                m40_float4 since, until;
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    since[r] = __builtin_amdgcn_exp2f(past[r] * f);
                    until[r] = __builtin_amdgcn_exp2f(end[r] - l[r]);
                }
                put4(&lds.qe[t_in][d], at4(&lds.q[t_in][d]) * since);
                put4(&lds.ks[t_in][d], at4(&lds.k[t_in][d]) * until);
            }
        }
        __syncthreads();
#pragma unroll
        for (int h = 0; h < 2; ++h) {               // decayed from the start, to the end
            const int d = d_in + 4 * h;
            put4(out + tile_at(t_in, slab + d, a.dp / 16u), at4(&lds.qe[t_in][d]) * at4(&lds.start[t_in >> 4][d]));
        }
#pragma unroll
        for (int h = 0; h < 2; ++h) {               // block `wave` of tokens, 16 dimensions
            const int d = h * 16 + li;
            m40_float4 y;
#pragma unroll
            for (int r = 0; r < 4; ++r) y[r] = lds.ks[wave * 16 + 4 * g + r][d] * lds.rest[wave][d];
            put4(out + a.at_k + (((slab / 16u + h) * 4u + wave) * 64 + lane) * 4, y);
        }
        {                                           // pairs of the block's own rows
            const int j = lane >> 2, d = (lane & 3) * 8;
            float kj[8], lj[8];
#pragma unroll
            for (int h = 0; h < 2; ++h) {
                const m40_float4 x = at4(&lds.k[wave * 16 + j][d + 4 * h]), y = at4(&lds.l[wave * 16 + j][d + 4 * h]);
#pragma unroll
                for (int r = 0; r < 4; ++r) { kj[4 * h + r] = x[r]; lj[4 * h + r] = y[r]; }
            }
#pragma unroll
            for (int t = 1; t < 16; ++t) {
#pragma unroll
                for (int h = 0; h < 2; ++h) {
                    const m40_float4 qt = at4(&lds.q[wave * 16 + t][d + 4 * h]), lt = at4(&lds.l[wave * 16 + t - 1][d + 4 * h]);
#pragma unroll
                    for (int r = 0; r < 4; ++r) own[t] = fmaf(qt[r], kj[4 * h + r] * __builtin_amdgcn_exp2f(fminf(lt[r] - lj[4 * h + r], 0.0f)), own[t]);
                }
                if (t & 1) stay();                  // operands of two rows at a time in registers
            }
        }
#pragma unroll
        for (int i = 0; i < 2; ++i)
#pragma unroll
            for (int h = 0; h < 2; ++h) {
                const int d = h * 16 + 4 * g, x = x_of[i], y = y_of[i];
                // decays of the blocks between: at most the second and the third
                const float f1 = y < 1 && x > 1 ? 1.0f : 0.0f, f2 = y < 2 && x > 2 ? 1.0f : 0.0f;
                m40_float4 f = at4(&lds.whole[1][d]) * f1 + at4(&lds.whole[2][d]) * f2;
#pragma unroll
                for (int r = 0; r < 4; ++r) f[r] = __builtin_amdgcn_exp2f(f[r]);
                off[i] = mma4(at4(&lds.ks[y * 16 + li][d]), at4(&lds.qe[x * 16 + li][d]) * f, off[i]);
            }
        __syncthreads();
    }
    {
        const int j = lane >> 2;
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            float y = own[t];
            y += m40_dpp_f<M40_DPP_XOR1>(y);
            y += m40_dpp_f<M40_DPP_XOR2>(y);
            if ((lane & 3) == (t & 3) && j != t) out[a.at_p + tile_at(wave * 16 + t, wave * 16 + (j & 12), 4u) + (j & 3)] = j < t ? y : 0.0f;
        }
        bonus += m40_dpp_f<M40_DPP_XOR1>(bonus);
        bonus += m40_dpp_f<M40_DPP_XOR2>(bonus);
        if ((lane & 3) == 0) out[a.at_p + tile_at(t_in, t_in & 60, 4u) + (t_in & 3)] = bonus;
#pragma unroll
        for (int i = 0; i < 2; ++i)
            if (wave + 4 * i < 6) put4(out + a.at_p + ((x_of[i] * 4 + y_of[i]) * 64 + lane) * 4, off[i]);
    }
    for (uint32_t x = wave; x < a.vt * 4u; x += 4u) {
        const uint32_t v = x % a.vt * 16u + li;
        m40_float4 y;
#pragma unroll
        for (uint32_t r = 0; r < 4; ++r) {
            const uint32_t t = x / a.vt * 16u + 4u * g + r;
            const float u = a.v[(size_t)row_of(t) * a.ld + head * a.vdim + (v < a.vdim ? v : 0u)];
            y[r] = t < n && v < a.vdim ? u : 0.0f;
        }
        put4(out + a.at_u + (x * 64 + lane) * 4, y);
    }
}

// ---- the walk ---------------------------------------------------------------------------------------------------------------------------
// Wave w holds key dimensions 16 DT w .. of 16 value columns.  A chunk's operands are requested SETS - 1 chunks ahead.
template <int WAVES, int DT, int SETS, M40MemoryRule RULE>
__global__ __launch_bounds__(WAVES * 64) void memory_walk_kernel(M40MemoryArgs a) {
    constexpr bool DELTA = RULE == kM40Delta;
    __shared__ m40_float4 part[DELTA ? WAVES : 1][4][64], whole[4][64];            // what the waves read of S; u
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), g = lane >> 4, li = lane & 15;
    const uint32_t p = blockIdx.x / a.heads, head = blockIdx.x % a.heads, V = blockIdx.y, v = V * 16u + li;
    const uint32_t *portion = a.portions + 4 * p, row0 = portion[0], end = row0 + portion[1];
    const uint32_t chunks = (end - 1u) / kChunk - row0 / kChunk + 1u;
    float* state = a.state + ((size_t)portion[2] * a.heads + head) * a.head_floats;
    float* own = state + (v < a.vdim ? v : (size_t)a.dim * a.v4);                  // column v of S; behind the last, n
    const size_t step_d = v < a.vdim ? a.v4 : 1u;
    const bool stored = v < a.vdim || (RULE == kM40Memory && v == a.vdim), fresh = a.row_pos[row0] == 0u;
    m40_float4 S[DT];
#pragma unroll
    for (int i = 0; i < DT; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const uint32_t d = (wave * DT + i) * 16 + 4 * g + r;
            S[i][r] = stored && !fresh && d < a.dim ? own[d * step_d] : 0.0f;
        }
    float* block = block_of(a, a.chunk_base[p], head);
    const size_t next = (size_t)a.heads * a.block;
    // u: of the delta rule, tile `wave` only (waves 0 to 3)
    struct Operands { m40_float4 w[DELTA ? 4 : 1][DT], k[DT][4], u[DELTA ? 1 : 4], decay[DT]; } set[SETS];
    auto load = [&](Operands& f, uint32_t c) __attribute__((always_inline)) {
        const float* b = block + (c < chunks ? c : chunks - 1u) * next;
        if (DELTA) {
#pragma unroll
            for (int t = 0; t < 4; ++t)
#pragma unroll
                for (int i = 0; i < DT; ++i) f.w[DELTA ? t : 0][i] = at4(b + a.at_w + ((t * (a.dp / 16u) + wave * DT + i) * 64 + lane) * 4);
            f.u[0] = at4(b + a.at_u + (((wave & 3) * a.vt + V) * 64 + lane) * 4);
        } else {
#pragma unroll
            for (int t = 0; t < 4; ++t) f.u[DELTA ? 0 : t] = at4(b + a.at_u + ((t * a.vt + V) * 64 + lane) * 4);
        }
#pragma unroll
        for (int i = 0; i < DT; ++i) {
            f.decay[i] = at4(b + a.at_decay + (wave * DT + i) * 16 + 4 * g);
#pragma unroll
            for (int t = 0; t < 4; ++t) f.k[i][t] = at4(b + a.at_k + (((wave * DT + i) * 4 + t) * 64 + lane) * 4);
        }
    };
    auto step = [&](const Operands& f, uint32_t c) __attribute__((always_inline)) {
        float* b = block + c * next;
#pragma unroll
        for (int i = 0; i < DT; ++i) put4(b + a.at_s + (((wave * DT + i) * a.vt + V) * 64 + lane) * 4, S[i]);
        m40_float4 u[4];
        if (DELTA) {
#pragma unroll
            for (int t = 0; t < 4; ++t) {
                m40_float4 read = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int i = 0; i < DT; ++i) read = mma4(f.w[DELTA ? t : 0][i], S[i], read);
                part[DELTA ? wave : 0][t][lane] = read;
            }
            m40_wait_and_meet<63>();
            if (wave < 4) {
                m40_float4 x = f.u[0];
#pragma unroll
                for (int w = 0; w < WAVES; ++w) x -= part[DELTA ? w : 0][wave][lane];
                whole[wave][lane] = x;
                put4(b + a.at_u + ((wave * a.vt + V) * 64 + lane) * 4, x);
            }
            m40_wait_and_meet<63>();
#pragma unroll
            for (int t = 0; t < 4; ++t) u[t] = whole[t][lane];
        } else {
#pragma unroll
            for (int t = 0; t < 4; ++t) u[t] = f.u[DELTA ? 0 : t];
        }
#pragma unroll
        for (int i = 0; i < DT; ++i) {
            S[i] *= f.decay[i];
#pragma unroll
            for (int t = 0; t < 4; ++t) S[i] = mma4(f.k[i][t], u[t], S[i]);
        }
    };
#pragma unroll
    for (int i = 0; i + 1 < SETS; ++i) load(set[i], i);
    for (uint32_t c = 0; c < chunks; c += SETS) {
#pragma unroll
        for (int i = 0; i < SETS; ++i) {
            if (c + i >= chunks) break;
            load(set[(i + SETS - 1) % SETS], c + i + SETS - 1);
            __builtin_amdgcn_sched_barrier(0);
            step(set[i], c + i);
        }
    }
    if (!stored) return;
#pragma unroll
    for (int i = 0; i < DT; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const uint32_t d = (wave * DT + i) * 16 + 4 * g + r;
            if (d < a.dim) own[d * step_d] = S[i][r];
        }
}

// ---- outputs: wave w takes the chunk's rows 16 w ..; VT: the most column tiles
template <int VT, M40MemoryRule RULE>
__global__ __launch_bounds__(256) void memory_outputs_kernel(M40MemoryArgs a) {
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), g = lane >> 4, li = lane & 15;
    const Chunk c(a, blockIdx.x);
    const uint32_t head = blockIdx.y;
    if (wave * 16 >= (int)c.n) return;
    const float* block = block_of(a, blockIdx.x, head);
    const int vt = (int)a.vt, t = wave * 16 + li;
    m40_float4 o[VT];
#pragma unroll
    for (int j = 0; j < VT; ++j) o[j] = m40_float4{0.f, 0.f, 0.f, 0.f};
    // 16 key dimensions of the state a step, then 16 of the chunk's tokens; operands are requested a step ahead
    const int d_steps = (int)(a.dim + 15u) / 16, steps = d_steps + wave + 1;
    struct Operands { m40_float4 x, y[VT]; } even, odd;
    auto load = [&](Operands& f, int n) __attribute__((always_inline)) {
        n = n < steps ? n : steps - 1;
        const bool state = n < d_steps;
        const float* tiles = block + (state ? a.at_s + n * vt * 256 : a.at_u + (n - d_steps) * vt * 256) + lane * 4;
        f.x = at4((state ? block + (wave * (int)(a.dp / 16u) + n) * 256 : block + a.at_p + (wave * 4 + n - d_steps) * 256) + lane * 4);
#pragma unroll
        for (int j = 0; j < VT; ++j) f.y[j] = at4(tiles + (j < vt ? j : vt - 1) * 256);
    };
    auto add = [&](const Operands& f) __attribute__((always_inline)) {
#pragma unroll
        for (int j = 0; j < VT; ++j)
            if (j < vt) o[j] = mma4(f.y[j], f.x, o[j]);
    };
    load(even, 0);
    for (int n = 0; n < steps; n += 2) {
        load(odd, n + 1);
        __builtin_amdgcn_sched_barrier(0);
        add(even);
        if (n + 1 >= steps) break;
        load(even, n + 2);
        __builtin_amdgcn_sched_barrier(0);
        add(odd);
    }
    const int vdim = (int)a.vdim;
    float f = 1.0f;
    if (RULE == kM40Memory) {                       // column vdim: n . q
        float x = 0.0f;
#pragma unroll
        for (int j = 0; j < VT; ++j)
            if (j == vdim / 16) {
#pragma unroll
                for (int r = 0; r < 4; ++r)
                    if (r == vdim % 4) {
                        x = o[j][r];
                        if (g == vdim % 16 / 4) o[j][r] = 0.0f;
                    }
            }
        x = __shfl(x, vdim % 16 / 4 * 16 + li);
        f = 1.0f / (fmaxf(fabsf(x), expf(-block[a.at_gate + 128 + t])) + 1e-6f);
    }
    float ss = 0.0f;
#pragma unroll
    for (int j = 0; j < VT; ++j) {
        o[j] *= f;
        ss += o[j][0] * o[j][0] + o[j][1] * o[j][1] + o[j][2] * o[j][2] + o[j][3] * o[j][3];
    }
    ss = m40_add_xor32(m40_add_xor16(ss));
    if (t >= (int)c.n) return;
    const float inv = a.out_factor / sqrtf(ss / (float)vdim + a.eps);
    const uint32_t row = c.row0 + t;
    const float *gate = a.gate + (size_t)row * a.ld_gate + head * a.vdim, *norm = a.norm + head * a.norm_stride;
    const bool vec = vdim % 4 == 0 && a.ld_gate % 4u == 0 && m40_aligned16(a.gate) && m40_aligned16(a.norm);
#pragma unroll
    for (int j = 0; j < VT; ++j) {
        const int v = j * 16 + 4 * g;
        if (j >= vt || v >= vdim) continue;
        const m40_float4 z = m40_load4(gate + v, vdim - v, vec), w = m40_load4(norm + v, vdim - v, vec);
        m40_float4 y;
#pragma unroll
        for (int r = 0; r < 4; ++r) y[r] = o[j][r] * inv * w[r] * (RULE == kM40Mixing ? m40_silu(z[r]) : m40_sigmoid(z[r]));
        m40_store_packed<m40_bf16>(static_cast<m40_bf16*>(a.out), (int)row, (int)(a.out_col + head * a.vdim) + v, (long)a.ld_out, y, vdim - v, vdim % 4 == 0 && a.out_col % 4u == 0);
    }
}

template <int WAVES, int DT, int SETS, M40MemoryRule RULE>
void walk(hipStream_t stream, const M40MemoryArgs& a, uint32_t n_portions) {
    memory_walk_kernel<WAVES, DT, SETS, RULE><<<dim3(n_portions * a.heads, a.vt), WAVES * 64, 0, stream>>>(a);
}
template <M40MemoryRule RULE>
int chunked(hipStream_t stream, const M40MemoryArgs& a, uint32_t n_portions, uint32_t n_chunks) {
    const bool vec = a.dim % 4u == 0 && a.ld % 4u == 0 && a.ld_a % 4u == 0 && m40_aligned16(a.q) && m40_aligned16(a.k) && m40_aligned16(a.a) && m40_aligned16(a.dt_bias);
    const dim3 grid(n_chunks, a.heads);
    constexpr bool DELTA = RULE == kM40Delta;
    if constexpr (RULE == kM40Mixing) {
        if (vec && m40_aligned16(a.bonus)) mixing_prepare_kernel<true><<<grid, 256, 0, stream>>>(a);
        else mixing_prepare_kernel<false><<<grid, 256, 0, stream>>>(a);
    } else if constexpr (DELTA) {
        static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(delta_prepare_kernel<true>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)sizeof(DeltaLds)),
                                attr2 = hipFuncSetAttribute(reinterpret_cast<const void*>(delta_prepare_kernel<false>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)sizeof(DeltaLds));
        if (attr != hipSuccess || attr2 != hipSuccess) return -2;
        if (vec) delta_prepare_kernel<true><<<grid, 256, sizeof(DeltaLds), stream>>>(a);
        else delta_prepare_kernel<false><<<grid, 256, sizeof(DeltaLds), stream>>>(a);
    } else {
        memory_scan_kernel<<<dim3(n_portions, a.heads), 1024, 0, stream>>>(a);
        if (vec) memory_prepare_kernel<true><<<grid, 256, 0, stream>>>(a);
        else memory_prepare_kernel<false><<<grid, 256, 0, stream>>>(a);
    }
    switch (a.dp / 64u) {
        case 1: walk<4, 1, 3, RULE>(stream, a, n_portions); break;
        case 2: walk<DELTA ? 8 : 4, DELTA ? 1 : 2, 3, RULE>(stream, a, n_portions); break;
        case 3: walk<12, 1, 2, RULE>(stream, a, n_portions); break;
        default: walk<8, 2, 2, RULE>(stream, a, n_portions); break;
    }
    if (a.vt <= 4u) memory_outputs_kernel<4, RULE><<<grid, 256, 0, stream>>>(a);
    else if (a.vt <= 8u) memory_outputs_kernel<8, RULE><<<grid, 256, 0, stream>>>(a);
    else if (a.vt <= 9u) memory_outputs_kernel<9, RULE><<<grid, 256, 0, stream>>>(a);
    else memory_outputs_kernel<17, RULE><<<grid, 256, 0, stream>>>(a);
    return hipGetLastError() == hipSuccess ? 0 : -2;
}

constexpr uint32_t kMost = 256;
// the parts of a block of scratch
void lay_out(M40MemoryArgs& a, M40MemoryRule rule) {
    a.dp = (a.dim + 63u) / 64u * 64u;
    a.vt = (a.vdim + (rule == kM40Memory ? 1u : 0u) + 15u) / 16u;
    uint32_t at = kChunk * a.dp;
    auto part = [&](uint32_t n) { const uint32_t x = at; at += n; return x; };
    a.at_k = part(kChunk * a.dp);
    a.at_p = part(kChunk * kChunk);
    a.at_u = part(kChunk * 16u * a.vt);
    a.at_decay = part(a.dp);
    a.at_s = part(a.dp * 16u * a.vt);
    a.at_w = part(rule == kM40Delta ? kChunk * a.dp : 0u);
    a.at_gate = part(rule == kM40Memory ? 256u : 0u);
    a.block = at;
}
uint64_t state_floats(M40MemoryRule rule, uint32_t dim, uint32_t vdim) {
    const uint64_t s = (uint64_t)dim * ((vdim + 3u) & ~3u);
    return rule != kM40Memory ? s : s + ((dim + 3u) & ~3u) + 4u;
}

// what the rules' structs have in common
template <class P>
int run(M40llmCudaContext* ctx, M40MemoryArgs& a, const P& p, uint32_t vdim, M40MemoryRule rule, uint32_t stream_kind) {
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    if (p.act_dtype > 1u || p.heads == 0 || p.heads > 65535u || p.n_portions == 0 || !m40llm_ext_memory_serves(p.dim, vdim) || p.ld_out % 32u != 0 ||
        p.ld_out < p.out_col + (uint64_t)p.heads * vdim || !m40_aligned16(p.state) || !m40_aligned16(p.out))
        return -3;
    a.heads = p.heads; a.dim = p.dim; a.vdim = vdim; a.v4 = (vdim + 3u) & ~3u;
    a.eps = p.eps; a.out_factor = p.out_factor;
    a.state = static_cast<float*>(p.state);
    a.head_floats = state_floats(rule, p.dim, vdim);
    a.out = p.out; a.ld_out = p.ld_out; a.out_col = p.out_col;
    a.portions = p.portions; a.chunk_base = p.chunk_base; a.chunks = p.chunks; a.row_pos = p.row_pos;
    a.scratch = static_cast<float*>(p.scratch);
    lay_out(a, rule);
    (void)hipGetLastError();
    if (!p.chunked) return m40_launch_memory_serial(stream, a, rule, p.act_dtype, p.n_portions);
    if (p.act_dtype != M40LLM_ACT_BF16 || !p.chunk_base || !p.chunks || p.n_chunks == 0 || !p.scratch || !m40_aligned16(p.scratch) ||
        p.scratch_bytes < (uint64_t)p.n_chunks * p.heads * a.block * 4u)
        return -4;
    switch (rule) {
        case kM40Delta: return chunked<kM40Delta>(stream, a, p.n_portions, p.n_chunks);
        case kM40Mixing: return chunked<kM40Mixing>(stream, a, p.n_portions, p.n_chunks);
        default: return chunked<kM40Memory>(stream, a, p.n_portions, p.n_chunks);
    }
}

}  // namespace

extern "C" {

int m40llm_ext_memory_serves(uint32_t dim, uint32_t vdim) { return dim >= 1u && dim <= kMost && vdim >= 1u && vdim <= kMost; }
uint64_t m40llm_ext_matrix_memory_state_floats(uint32_t dim, uint32_t vdim) { return state_floats(kM40Memory, dim, vdim); }
uint64_t m40llm_ext_channel_delta_state_floats(uint32_t dim, uint32_t vdim) { return state_floats(kM40Delta, dim, vdim); }
uint64_t m40llm_ext_memory_scratch_bytes(uint32_t rule, uint32_t n_chunks, uint32_t heads, uint32_t dim, uint32_t vdim) {
    M40MemoryArgs a{};
    a.dim = dim; a.vdim = vdim;
    lay_out(a, (M40MemoryRule)rule);
    return (uint64_t)n_chunks * heads * a.block * 4u;
}

int m40llm_ext_matrix_memory_async(M40llmCudaContext* ctx, const M40llmMatrixMemory* m, uint32_t stream_kind) {
    if (!ctx || !m || !m->proj || !m->i_bias || !m->f_bias || !m->norm || !m->state || !m->out || !m->portions || !m->row_pos) return -1;
    const uint64_t q = (uint64_t)m->heads * m->dim, v = (uint64_t)m->heads * m->vdim;
    if (m->ld_proj < m->q_col + q || m->ld_proj < m->k_col + q || m->ld_proj < m->v_col + v || m->ld_proj < m->g_col + v || m->ld_proj < (uint64_t)m->i_col + m->heads ||
        m->ld_proj < (uint64_t)m->f_col + m->heads || !(m->cap > 0.0f))
        return -3;
    M40MemoryArgs a{};
    const float* x = static_cast<const float*>(m->proj);
    a.share = 1u;
    a.q = x + m->q_col; a.k = x + m->k_col; a.v = x + m->v_col; a.ld = m->ld_proj;
    a.i = x + m->i_col; a.f = x + m->f_col; a.i_bias = static_cast<const float*>(m->i_bias); a.f_bias = static_cast<const float*>(m->f_bias);
    a.cap = m->cap;
    a.norm = static_cast<const float*>(m->norm); a.norm_stride = m->vdim;
    a.gate = x + m->g_col; a.ld_gate = m->ld_proj;
    a.q_factor = m->q_factor;
    return run(ctx, a, *m, m->vdim, kM40Memory, stream_kind);
}

int m40llm_ext_channel_delta_async(M40llmCudaContext* ctx, const M40llmChannelDelta* m, uint32_t stream_kind) {
    if (!ctx || !m || !m->qkv || !m->low || !m->beta || !m->A_log || !m->dt_bias || !m->norm || !m->state || !m->out || !m->portions || !m->row_pos) return -1;
    if (m->kv_heads == 0 || m->heads % m->kv_heads != 0 || m->ld_qkv < 2ull * m->kv_heads * m->dim + (uint64_t)m->heads * m->vdim ||
        m->ld_low < m->a_col + (uint64_t)m->heads * m->dim || m->ld_low < m->g_col + (uint64_t)m->heads * m->vdim || m->ld_beta < m->heads)
        return -3;
    M40MemoryArgs a{};
    const float *x = static_cast<const float*>(m->qkv), *low = static_cast<const float*>(m->low);
    a.share = m->heads / m->kv_heads;
    a.q = x; a.k = x + (size_t)m->kv_heads * m->dim; a.v = x + 2u * (size_t)m->kv_heads * m->dim; a.ld = m->ld_qkv;
    a.a = low + m->a_col; a.ld_a = m->ld_low;
    a.beta = static_cast<const float*>(m->beta); a.ld_beta = m->ld_beta;
    a.A_log = static_cast<const float*>(m->A_log); a.dt_bias = static_cast<const float*>(m->dt_bias);
    a.norm = static_cast<const float*>(m->norm); a.norm_stride = 0;
    a.gate = low + m->g_col; a.ld_gate = m->ld_low;
    a.q_factor = m->q_factor;
    return run(ctx, a, *m, m->vdim, kM40Delta, stream_kind);
}

int m40llm_ext_time_mixing_async(M40llmCudaContext* ctx, const M40llmTimeMixing* m, uint32_t stream_kind) {
    if (!ctx || !m || !m->rkv || !m->decay || !m->w0 || !m->u || !m->norm || !m->state || !m->out || !m->portions || !m->row_pos) return -1;
    const uint64_t cols = (uint64_t)m->heads * m->dim;
    if (m->ld_rkv < m->r_col + cols || m->ld_rkv < m->k_col + cols || m->ld_rkv < m->v_col + cols || m->ld_rkv < m->g_col + cols || m->ld_decay < cols) return -3;
    M40MemoryArgs a{};
    const float* x = static_cast<const float*>(m->rkv);
    a.share = 1u;
    a.q = x + m->r_col; a.k = x + m->k_col; a.v = x + m->v_col; a.ld = m->ld_rkv;
    a.q_factor = 1.0f;
    a.a = static_cast<const float*>(m->decay); a.ld_a = m->ld_decay;
    a.dt_bias = static_cast<const float*>(m->w0); a.bonus = static_cast<const float*>(m->u);
    a.norm = static_cast<const float*>(m->norm); a.norm_stride = m->dim;
    a.gate = x + m->g_col; a.ld_gate = m->ld_rkv;
    return run(ctx, a, *m, m->dim, kM40Mixing, stream_kind);
}

}  // extern "C"
