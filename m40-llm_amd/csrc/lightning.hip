// Linear attention with one decay per head: S <- decay S + k v^T, o = S^T q.  Stepped form (STEPS, state space layers): the decay and the weight of
// k v^T come from the token's step size, heads share queries and keys, and o has a direct part, skip v.
//
// lightning_serial_kernel   token after token in f32, a workgroup a portion, head and 32 value columns: decoded tokens, and every portion in
//                           f32.  A thread holds S for four columns and every 32nd key dimension.
// lightning_steps_kernel    bf16 portions, stepped: step sizes and sums of log decays of all chunks
// lightning_states_kernel   bf16 portions, the walk over the 64-row groups ("chunks") of a portion: a workgroup holds S for 32 key
//                           dimensions x 64 value columns of a head, leaves it as it is before each chunk, and adds the chunk's keys and values
// lightning_outputs_kernel  bf16 portions, all chunks at once: what the state before the chunk gives, plus the chunk's own keys
//
// Chunks are groups of 64 rows of the step, not of the portion, so that rows lie in whole operand tiles; tokens of other portions in a
// chunk have weight zero.  Everything that is not a projection stays in f32: the state and the decayed weights and values enter the matrix
// instruction as two bf16 parts (value and remainder), which keeps 16 bits of them.
#include "memory_rules.hpp"

namespace {

constexpr uint32_t kMostDim = 256;
constexpr int kChunk = 64;

struct LightArgs {
    M40llmLightning l;
    uint32_t d_pad, v_pad, kv_heads, share;        // share: heads that use one query / key head
    float* steps;                                  // [chunk][head][kStepFloats]
    __device__ float* state(uint32_t slot, uint32_t head) const { return static_cast<float*>(l.state) + ((size_t)slot * l.heads + head) * l.dim * v_pad; }
};

// Of a chunk and head: weight of every token's k v^T in the state at the chunk's end [64], sums of log2 decays since the portion's first token in the
// chunk [64], step sizes [64] (weights and steps zero outside the portion), the whole chunk's decay
constexpr int kStepFloats = 256, kAtSum = 64, kAtStep = 128, kAtWhole = 192;
__device__ __forceinline__ float step_size(const M40llmLightning& l, uint32_t row, uint32_t head) {
    return m40_softplus(static_cast<const float*>(l.step_logits)[(size_t)row * l.ld_step + head] + static_cast<const float*>(l.step_bias)[head]);
}
// log2 of a token's decay; what is below this is nothing in f32
__device__ __forceinline__ float step_decay(float rate, float step) { return fmaxf(-rate * step * kM40Log2e, -160.0f); }

__global__ __launch_bounds__(256) void lightning_steps_kernel(LightArgs a) {
    const uint32_t lane = threadIdx.x & 63u, head = blockIdx.y * 4u + (threadIdx.x >> 6);
    if (head >= a.l.heads) return;
    const uint32_t *portion = a.l.portions + 4 * a.l.chunks[2 * blockIdx.x], row = a.l.chunks[2 * blockIdx.x + 1] + lane;
    const bool in = row >= portion[0] && row < portion[0] + portion[1];
    const float z = step_size(a.l, in ? row : portion[0], head), step = in ? z : 0.0f;
    float sum = step_decay(expf(static_cast<const float*>(a.l.A_log)[head]), step);
#pragma unroll
    for (int d = 1; d < 64; d *= 2) {
        const float s = __shfl_up(sum, d);
        if ((int)lane >= d) sum += s;
    }
    const float end = __shfl(sum, 63);
    float* out = a.steps + ((size_t)blockIdx.x * a.l.heads + head) * kStepFloats + lane;
    out[0] = step * __builtin_amdgcn_exp2f(end - sum);
    out[kAtSum] = sum;
    out[kAtStep] = step;
    out[kAtWhole] = __builtin_amdgcn_exp2f(end);
}

__device__ __forceinline__ float decay_power(float log2_decay, int n) { return n == 0 ? 1.0f : __builtin_amdgcn_exp2f(log2_decay * (float)n); }

template <class T, uint32_t kMine, bool STEPS>       // kMine: key dimensions of a thread
__global__ __launch_bounds__(256) void lightning_serial_kernel(LightArgs a) {
    __shared__ m40_float4 sums[2][4][8];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, d0 = tid >> 3;
    const uint32_t* portion = a.l.portions + 4 * blockIdx.x;
    const uint32_t row0 = portion[0], n = portion[1], head = blockIdx.y, v0 = blockIdx.z * 32u + (tid & 7u) * 4u, dim = a.l.dim;
    const uint32_t k_tiles = (uint32_t)(a.l.ld_qkv >> 5), q_col = head / a.share * a.d_pad, k_col = (a.kv_heads + head / a.share) * a.d_pad, v_col = 2u * a.kv_heads * a.d_pad + head * a.v_pad + v0;
    const T* qkv = static_cast<const T*>(a.l.qkv);
    const float fixed = STEPS ? 0.0f : static_cast<const float*>(a.l.decay)[head], rate = STEPS ? expf(static_cast<const float*>(a.l.A_log)[head]) : 0.0f;
    const float skip = STEPS ? static_cast<const float*>(a.l.skip)[head] : 0.0f;
    float* state = a.state(portion[2], head) + v0;
    const bool fresh = a.l.row_pos[row0] == 0u;
    m40_float4 S[kMine];
#pragma unroll
    for (uint32_t i = 0; i < kMine; ++i) {
        const uint32_t d = d0 + 32u * i;
        S[i] = m40_float4{0.f, 0.f, 0.f, 0.f};
        if (d < dim && !fresh) S[i] = *reinterpret_cast<const m40_float4*>(state + (size_t)d * a.v_pad);
    }
    for (uint32_t t = 0; t < n; ++t) {
        const uint32_t row = row0 + t;
        const T* vp = qkv + m40_packed_at(row, v_col, k_tiles);
        const m40_float4 v = {M40Act<T>::to(vp[0]), M40Act<T>::to(vp[1]), M40Act<T>::to(vp[2]), M40Act<T>::to(vp[3])};
        m40_float4 o = {0.f, 0.f, 0.f, 0.f};
        const float step = STEPS ? step_size(a.l, row, head) : 1.0f, decay = STEPS ? expf(-rate * step) : fixed;
        const m40_float4 add = v * step;
#pragma unroll
        for (uint32_t i = 0; i < kMine; ++i) {
            const uint32_t d = d0 + 32u * i;
            if (d < dim) {
                const float k = M40Act<T>::to(qkv[m40_packed_at(row, k_col + d, k_tiles)]), q = M40Act<T>::to(qkv[m40_packed_at(row, q_col + d, k_tiles)]);
                S[i] = S[i] * decay + add * k;
                o += S[i] * q;
            }
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) o[r] = m40_sum_lanes_from<8>(o[r]);
        if (lane < 8u) sums[t & 1u][wave][lane] = o;
        __syncthreads();
        if (tid < 8u) {
            const m40_float4 y = sums[t & 1u][0][tid] + sums[t & 1u][1][tid] + sums[t & 1u][2][tid] + sums[t & 1u][3][tid] + v * skip;
            float* out = static_cast<float*>(a.l.o) + (size_t)row * a.l.ld_o + head * a.l.vdim + v0;
#pragma unroll
            for (uint32_t r = 0; r < 4u; ++r)
                if (v0 + r < a.l.vdim) out[r] = y[r];
        }
    }
#pragma unroll
    for (uint32_t i = 0; i < kMine; ++i) {
        const uint32_t d = d0 + 32u * i;
        if (d < dim) *reinterpret_cast<m40_float4*>(state + (size_t)d * a.v_pad) = S[i];
    }
}

// the 4 x 16 transposed read: of 16 lanes' addresses (four rows, four pieces of 4 columns each) lane i receives column i of the rows
__device__ __forceinline__ m40_bf16x8 read_columns(const uint8_t* p0, const uint8_t* p1) {
    typedef short s16x4 __attribute__((ext_vector_type(4)));
    typedef __attribute__((address_space(3))) s16x4* lds4_t;
    typedef short s16x8 __attribute__((ext_vector_type(8)));
    const s16x4 a = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds4_t)(p0));
    const s16x4 b = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds4_t)(p1));
    return __builtin_bit_cast(m40_bf16x8, s16x8{a.x, a.y, a.z, a.w, b.x, b.y, b.z, b.w});
}
// bytes of tokens tok0 .. tok0 + 3 of a 16-token operand tile, columns 16 c16 .. of its 32 (this lane's address for read_columns)
__device__ __forceinline__ uint32_t column_address(int li, int tok0, int c16) {
    const int d = c16 * 16 + (li & 3) * 4;
    return (uint32_t)((((d >> 3) * 16 + tok0 + (li >> 2)) * 8 + (d & 7)) * 2);
}
struct Parts { m40_bf16x8 hi, lo; };
__device__ __forceinline__ Parts two_parts(const float (&x)[8]) {
    Parts p;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
        p.hi[i] = static_cast<m40_bf16>(x[i]);
        p.lo[i] = static_cast<m40_bf16>(x[i] - static_cast<float>(p.hi[i]));
    }
    return p;
}

// Key dimensions and value columns of S are the rows and columns of the accumulators: a lane holds column lane % 16 and rows 4 g + r of two
// tiles, which as it is is an operand of 32 dimensions (dimension 16 t + 4 g + r at place 8 g + 4 t + r).
// Scratch: per chunk and head [32 dimensions][16 columns][2 parts] tiles.
template <bool STEPS>
__global__ __launch_bounds__(256) void lightning_states_kernel(LightArgs a) {
    typedef __attribute__((address_space(3))) void* lds_dst_t;
    typedef const __attribute__((address_space(1))) void* global_src_t;
    // per chunk: keys and values [4 row tiles][32, 2 x 32]; step weights (the same load by every wave)
    constexpr int kBufs = 4, kTiles = STEPS ? 13 : 12, kLoads = STEPS ? 4 : 3;
    __shared__ __align__(16) uint8_t lds[kBufs * kTiles * 1024];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), g = lane >> 4, li = lane & 15;
    const uint32_t* portion = a.l.portions + 4 * blockIdx.x;
    const uint32_t row0 = portion[0], n = portion[1], head = blockIdx.y;
    const uint32_t dt = a.d_pad / 32u, vt = a.v_pad / 32u, d32 = blockIdx.z % dt, v64 = blockIdx.z / dt;       // vt: 32-column tiles
    const uint32_t k_tiles = (uint32_t)(a.l.ld_qkv >> 5), k_tile = (a.kv_heads + head / a.share) * dt + d32, v_tile = 2u * a.kv_heads * dt + head * vt + v64 * 2u;
    const uint32_t first = row0 / kChunk, chunks = (row0 + n - 1u) / kChunk - first + 1u, last_rt = (row0 + n - 1u) / 16u;
    const uint32_t v_second = v64 * 2u + 1u < vt ? 1u : 0u;                        // a value half past the head's is the first again
    const m40_bf16* qkv = static_cast<const m40_bf16*>(a.l.qkv) + lane * 8;
    const float* steps = a.steps + ((size_t)a.l.chunk_base[blockIdx.x] * a.l.heads + head) * kStepFloats + lane * 4;
    auto issue = [&](int buf, uint32_t chunk) __attribute__((always_inline)) {     // three tiles a wave: its row tile of the chunk
        const uint32_t c = chunk < chunks ? chunk : chunks - 1u, rt = (first + c) * 4u + wave;
        const m40_bf16* src = qkv + (size_t)(rt < last_rt ? rt : last_rt) * k_tiles * kM40Tile;
        uint8_t* dst = lds + (buf * kTiles + wave * 3) * 1024;
        __builtin_amdgcn_global_load_lds((global_src_t)(src + (size_t)k_tile * kM40Tile), (lds_dst_t)(dst), 16, 0, 0);
        __builtin_amdgcn_global_load_lds((global_src_t)(src + (size_t)v_tile * kM40Tile), (lds_dst_t)(dst + 1024), 16, 0, 0);
        __builtin_amdgcn_global_load_lds((global_src_t)(src + (size_t)(v_tile + v_second) * kM40Tile), (lds_dst_t)(dst + 2048), 16, 0, 0);
        if (STEPS) __builtin_amdgcn_global_load_lds((global_src_t)(steps + (size_t)c * a.l.heads * kStepFloats), (lds_dst_t)(lds + (buf * kTiles + 12) * 1024), 16, 0, 0);
    };
#pragma unroll
    for (int i = 0; i < kBufs - 1; ++i) issue(i, i);
    const float log2_decay = STEPS ? 0.0f : static_cast<const float*>(a.l.log2_decay)[head];
    const uint32_t v16 = v64 * 4u + wave, v = v16 * 16u + li;          // this wave's value columns
    const bool wave_live = v16 * 16u < a.v_pad;
    float* state = a.state(portion[2], head);
    m40_float4 S[2];
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const uint32_t d = d32 * 32u + 16u * t + 4u * g + r;
            S[t][r] = wave_live && d < a.l.dim && a.l.row_pos[row0] != 0u ? state[(size_t)d * a.v_pad + v] : 0.0f;
        }
    m40_bf16* out = static_cast<m40_bf16*>(a.l.scratch) + ((size_t)a.l.chunk_base[blockIdx.x] * a.l.heads + head) * dt * vt * 4u * kM40Tile +
                    ((size_t)d32 * vt * 2u + v16) * 2u * kM40Tile + lane * 8;
    const size_t out_step = (size_t)a.l.heads * dt * vt * 4u * kM40Tile;
    float whole[2][8];                                                 // decay to the end of a whole chunk
#pragma unroll
    for (int h = 0; h < 2; ++h)
#pragma unroll
        for (int i = 0; i < 8; ++i) whole[h][i] = decay_power(log2_decay, kChunk - 1 - (32 * h + 8 * g + i));
    const float whole_chunk = decay_power(log2_decay, kChunk);
    int buf = 0;
    for (uint32_t c = 0; c < chunks; ++c) {
        // Chunk c has landed, and nobody reads the buffer before it any more.  Behind its own loads a wave has issued those of the two chunks
        // after it and, once the walk is under way, the two stores of each of three chunks.
        if (wave_live && c >= 3u) m40_wait_and_meet<kLoads * (kBufs - 2) + 6>();
        else m40_wait_and_meet<kLoads * (kBufs - 2)>();
        issue(buf == 0 ? kBufs - 1 : buf - 1, c + kBufs - 1);
        asm volatile("" ::: "memory");                                 // the stores stay behind these loads: they are counted
        __builtin_amdgcn_sched_barrier(0);
        float s8[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) s8[i] = S[i >> 2][i & 3];
        const Parts sp = two_parts(s8);
        if (wave_live) {
            *reinterpret_cast<m40_bf16x8*>(out + c * out_step) = sp.hi;
            *reinterpret_cast<m40_bf16x8*>(out + c * out_step + kM40Tile) = sp.lo;
        }
        const int base = (int)((first + c) * kChunk), lo = (int)row0 > base ? (int)row0 - base : 0, end = (int)(row0 + n) - base, hi = end < kChunk ? end : kChunk;
        const bool all = lo == 0 && hi == kChunk;
        const uint8_t* tiles = lds + buf * kTiles * 1024;
        const float* own = reinterpret_cast<const float*>(tiles + 12 * 1024);
        const float f = STEPS ? own[kAtWhole] : all ? whole_chunk : decay_power(log2_decay, hi - lo);
        S[0] *= f;
        S[1] *= f;
#pragma unroll
        for (int h = 0; h < 2; ++h) {                                  // 32 tokens: places 8 g ..
            const uint8_t* tile = tiles + (2 * h + (g >> 1)) * 3 * 1024;
            const int tok = (g & 1) * 8;
            const uint32_t at = column_address(li, tok, (int)(v16 & 1u)), half = ((v16 >> 1) & 1u) * 1024u;
            const m40_bf16x8 vf = read_columns(tile + 1024 + half + at, tile + 1024 + half + at + 4 * 16);
            float w[8];
            if (STEPS) {
                const m40_float4 w0 = *reinterpret_cast<const m40_float4*>(own + 32 * h + 8 * g), w1 = *reinterpret_cast<const m40_float4*>(own + 32 * h + 8 * g + 4);
#pragma unroll
                for (int i = 0; i < 8; ++i) {
                    const int j = 32 * h + 8 * g + i;       // rows outside the portion may hold anything
                    w[i] = all || (j >= lo && j < hi) ? static_cast<float>(vf[i]) * (i < 4 ? w0[i & 3] : w1[i & 3]) : 0.0f;
                }
            } else if (all) {
#pragma unroll
                for (int i = 0; i < 8; ++i) w[i] = static_cast<float>(vf[i]) * whole[h][i];
            } else {
#pragma unroll
                for (int i = 0; i < 8; ++i) {
                    const int j = 32 * h + 8 * g + i;
                    w[i] = j >= lo && j < hi ? static_cast<float>(vf[i]) * decay_power(log2_decay, hi - 1 - j) : 0.0f;
                }
            }
            const Parts vp = two_parts(w);
#pragma unroll
            for (int t = 0; t < 2; ++t) {
                const uint32_t kat = column_address(li, tok, t);
                const m40_bf16x8 kf = read_columns(tile + kat, tile + kat + 4 * 16);
                S[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, vp.hi, S[t], 0, 0, 0);
                S[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, vp.lo, S[t], 0, 0, 0);
            }
        }
        buf = buf == kBufs - 1 ? 0 : buf + 1;
    }
    m40_wait_and_meet<0>();
    if (!wave_live) return;
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const uint32_t d = d32 * 32u + 16u * t + 4u * g + r;
            if (d < a.l.dim) state[(size_t)d * a.v_pad + v] = S[t][r];
        }
}

// Wave w takes the chunk's rows 16 w ..; VT: 16-column value tiles.
template <int VT, bool STEPS>
__global__ __launch_bounds__(256) void lightning_outputs_kernel(LightArgs a) {
    typedef __attribute__((address_space(3))) void* lds_dst_t;
    typedef const __attribute__((address_space(1))) void* global_src_t;
    __shared__ __align__(16) float step_lds[STEPS ? kStepFloats : 4];
    extern __shared__ __align__(16) uint8_t lds[];           // states [d tiles][16-column tiles][2], values [4 row tiles][32-column tiles]
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), g = lane >> 4, li = lane & 15;
    const uint32_t* portion = a.l.portions + 4 * a.l.chunks[2 * blockIdx.x];
    const int base = (int)a.l.chunks[2 * blockIdx.x + 1], row0 = (int)portion[0], end = row0 + (int)portion[1];
    const uint32_t head = blockIdx.y;
    const int lo = row0 > base ? row0 - base : 0, hi = end - base < kChunk ? end - base : kChunk;
    const int dt = (int)a.d_pad / 32, vt = (int)a.v_pad / 32, last_rt = (end - 1) / 16;
    const uint32_t k_tiles = (uint32_t)(a.l.ld_qkv >> 5);
    const m40_bf16* qkv = static_cast<const m40_bf16*>(a.l.qkv) + lane * 8;
    const m40_bf16* states = static_cast<const m40_bf16*>(a.l.scratch) + ((size_t)blockIdx.x * a.l.heads + head) * dt * vt * 4 * kM40Tile + lane * 8;
    uint8_t* v_lds = lds + dt * vt * 4 * 1024;
    for (int i = wave; i < dt * vt * 4; i += 4)
        __builtin_amdgcn_global_load_lds((global_src_t)(states + (size_t)i * kM40Tile), (lds_dst_t)(lds + i * 1024), 16, 0, 0);
    auto row_tile = [&](int rt) { const int t = base / 16 + rt; return qkv + (size_t)(t < last_rt ? t : last_rt) * k_tiles * kM40Tile; };
    for (int i = 0; i < vt; ++i)
        __builtin_amdgcn_global_load_lds((global_src_t)(row_tile(wave) + (size_t)(2 * a.kv_heads * dt + head * vt + i) * kM40Tile), (lds_dst_t)(v_lds + (wave * vt + i) * 1024), 16, 0, 0);
    if (STEPS && wave == 0)
        __builtin_amdgcn_global_load_lds((global_src_t)(a.steps + ((size_t)blockIdx.x * a.l.heads + head) * kStepFloats + lane * 4), (lds_dst_t)(step_lds), 16, 0, 0);
    const float log2_decay = STEPS ? 0.0f : static_cast<const float*>(a.l.log2_decay)[head], skip = STEPS ? static_cast<const float*>(a.l.skip)[head] : 0.0f;
    m40_float4 o[VT];
#pragma unroll
    for (int j = 0; j < VT; ++j) o[j] = m40_float4{0.f, 0.f, 0.f, 0.f};
    // scores of this wave's queries with the keys of row tiles 0 .. wave
    m40_float4 s[4];
#pragma unroll
    for (int t = 0; t < 4; ++t) s[t] = m40_float4{0.f, 0.f, 0.f, 0.f};
    const m40_bf16* q_tiles = row_tile(wave) + (size_t)(head / a.share) * dt * kM40Tile;
    for (int k = 0; k < dt; ++k) {
        const m40_bf16x8 qf = *reinterpret_cast<const m40_bf16x8*>(q_tiles + (size_t)k * kM40Tile);
#pragma unroll
        for (int t = 0; t < 4; ++t)
            if (t <= wave) {
                const m40_bf16x8 kf = *reinterpret_cast<const m40_bf16x8*>(row_tile(t) + (size_t)((a.kv_heads + head / a.share) * dt + k) * kM40Tile);
                s[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf, s[t], 0, 0, 0);
            }
    }
    m40_wait_and_meet<0>();
    // what came before the chunk, operands of 32 key dimensions in the states' order
    for (int k = 0; k < dt; ++k) {
        typedef uint32_t u32x2 __attribute__((ext_vector_type(2)));
        typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
        const m40_bf16* tile = q_tiles - lane * 8 + (size_t)k * kM40Tile;
        const u32x2 q0 = *reinterpret_cast<const u32x2*>(tile + ((g >> 1) * 16 + li) * 8 + 4 * (g & 1));
        const u32x2 q1 = *reinterpret_cast<const u32x2*>(tile + ((2 + (g >> 1)) * 16 + li) * 8 + 4 * (g & 1));
        const m40_bf16x8 qf = __builtin_bit_cast(m40_bf16x8, u32x4{q0.x, q0.y, q1.x, q1.y});
        const uint8_t* st = lds + k * vt * 4 * 1024 + lane * 16;
#pragma unroll
        for (int j = 0; j < VT; ++j)
            if (j < 2 * vt) {
                o[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf, *reinterpret_cast<const m40_bf16x8*>(st + j * 2048), o[j], 0, 0, 0);
                o[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf, *reinterpret_cast<const m40_bf16x8*>(st + j * 2048 + 1024), o[j], 0, 0, 0);
            }
    }
    float f[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        const int i = wave * 16 + 4 * g + r;
        f[r] = i < lo ? 0.0f : STEPS ? __builtin_amdgcn_exp2f(step_lds[kAtSum + i]) : decay_power(log2_decay, i - lo + 1);
    }
#pragma unroll
    for (int j = 0; j < VT; ++j)
#pragma unroll
        for (int r = 0; r < 4; ++r) o[j][r] *= f[r];
    // the chunk's own keys up to each row
#pragma unroll
    for (int h = 0; h < 2; ++h) {
        if (2 * h > wave) continue;
        float w[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            const int j = 32 * h + 16 * (i >> 2) + 4 * g + (i & 3), q = wave * 16 + li;
            const float x = s[2 * h + (i >> 2)][i & 3];
            if (STEPS) w[i] = j <= q && j >= lo && j < hi ? fmaf(x * __builtin_amdgcn_exp2f(step_lds[kAtSum + q] - step_lds[kAtSum + j]), step_lds[kAtStep + j], j == q ? skip : 0.0f) : 0.0f;
            else w[i] = j <= q && j >= lo ? x * decay_power(log2_decay, q - j) : 0.0f;
        }
        const Parts p = two_parts(w);
        const uint8_t* t0 = v_lds + (2 * h) * vt * 1024;
        const uint8_t* t1 = t0 + vt * 1024;
#pragma unroll
        for (int j = 0; j < VT; ++j)
            if (j < 2 * vt) {
                const uint32_t at = (uint32_t)(j >> 1) * 1024u + column_address(li, 4 * g, j & 1);
                const m40_bf16x8 vf = read_columns(t0 + at, t1 + at);
                o[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(p.hi, vf, o[j], 0, 0, 0);
                o[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(p.lo, vf, o[j], 0, 0, 0);
            }
    }
    float* out = static_cast<float*>(a.l.o) + head * a.l.vdim;
#pragma unroll
    for (int j = 0; j < VT; ++j)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int i = wave * 16 + 4 * g + r;
            const uint32_t v = (uint32_t)(j * 16 + li);
            if (i >= lo && i < hi && v < a.l.vdim) out[(size_t)(base + i) * a.l.ld_o + v] = o[j][r];
        }
}

template <class T, bool STEPS>
int launch_serial(hipStream_t stream, const LightArgs& a) {
    const dim3 grid(a.l.n_portions, a.l.heads, a.v_pad / 32u);
    if (a.l.dim <= 64u) lightning_serial_kernel<T, 2, STEPS><<<grid, 256, 0, stream>>>(a);
    else if (a.l.dim <= 128u) lightning_serial_kernel<T, 4, STEPS><<<grid, 256, 0, stream>>>(a);
    else lightning_serial_kernel<T, 8, STEPS><<<grid, 256, 0, stream>>>(a);
    return hipGetLastError() == hipSuccess ? 0 : -2;
}

constexpr int kLdsMax = 160 * 1024, kLdsDynamic = kLdsMax - kStepFloats * 4;
template <int VT, bool STEPS>
int launch_outputs(hipStream_t stream, const LightArgs& a) {
    static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(lightning_outputs_kernel<VT, STEPS>), hipFuncAttributeMaxDynamicSharedMemorySize,
                                                       STEPS ? kLdsDynamic : kLdsMax);
    if (attr != hipSuccess) return -2;
    const int dt = (int)a.d_pad / 32, vt = (int)a.v_pad / 32;
    lightning_outputs_kernel<VT, STEPS><<<dim3(a.l.n_chunks, a.l.heads), 256, (dt * vt * 4 + 4 * vt) * 1024, stream>>>(a);
    return hipGetLastError() == hipSuccess ? 0 : -2;
}
uint64_t state_bytes(uint32_t n_chunks, uint32_t heads, uint32_t dim, uint32_t vdim) { return (uint64_t)n_chunks * heads * ((dim + 31u) / 32u) * ((vdim + 31u) / 32u) * 4096u; }

template <bool STEPS>
int launch_chunked(hipStream_t stream, const LightArgs& a) {
    if (STEPS) lightning_steps_kernel<<<dim3(a.l.n_chunks, (a.l.heads + 3u) / 4u), 256, 0, stream>>>(a);
    lightning_states_kernel<STEPS><<<dim3(a.l.n_portions, a.l.heads, a.d_pad / 32u * ((a.v_pad + 63u) / 64u)), 256, 0, stream>>>(a);
    if (hipGetLastError() != hipSuccess) return -2;
    if (a.v_pad <= 64u) return launch_outputs<4, STEPS>(stream, a);
    if (a.v_pad <= 128u) return launch_outputs<8, STEPS>(stream, a);
    return launch_outputs<16, STEPS>(stream, a);
}

}  // namespace

extern "C" {

int m40llm_ext_lightning_serves(uint32_t dim, uint32_t vdim) { return dim >= 1u && dim <= kMostDim && vdim >= 1u && vdim <= kMostDim; }
uint64_t m40llm_ext_lightning_scratch_bytes(uint32_t n_chunks, uint32_t heads, uint32_t dim, uint32_t vdim) {
    return state_bytes(n_chunks, heads, dim, vdim) + (uint64_t)n_chunks * heads * kStepFloats * 4u;
}

int m40llm_ext_lightning_async(M40llmCudaContext* ctx, const M40llmLightning* l, uint32_t stream_kind) {
    if (!ctx || !l || !l->qkv || (l->step_logits ? !l->step_bias || !l->A_log || !l->skip : !l->decay || !l->log2_decay) || !l->state || !l->o || !l->portions || !l->row_pos)
        return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    LightArgs a{*l, (l->dim + 31u) / 32u * 32u, (l->vdim + 31u) / 32u * 32u, l->kv_heads ? l->kv_heads : l->heads, 1u, nullptr};
    if (l->act_dtype > 1u || l->heads == 0 || l->heads > 65535u || l->heads % a.kv_heads != 0 || l->n_portions == 0 || !m40llm_ext_lightning_serves(l->dim, l->vdim) ||
        l->ld_qkv % 32u != 0 || l->ld_qkv < 2ull * a.kv_heads * a.d_pad + (uint64_t)l->heads * a.v_pad || l->ld_o < (uint64_t)l->heads * l->vdim ||
        (l->step_logits && l->ld_step < l->heads) || !m40_aligned16(l->qkv) || !m40_aligned16(l->state))
        return -3;
    a.share = l->heads / a.kv_heads;
    const bool steps = l->step_logits != nullptr;
    (void)hipGetLastError();
    // the states of a head fit LDS together with a chunk's values up to 128 x 256 or 256 x 128
    const uint32_t tiles = a.d_pad / 32u * (a.v_pad / 32u) * 4u + 4u * (a.v_pad / 32u);
    if (!l->chunked || tiles * 1024u > (uint32_t)(steps ? kLdsDynamic : kLdsMax)) {
        if (l->act_dtype == M40LLM_ACT_F32) return steps ? launch_serial<float, true>(stream, a) : launch_serial<float, false>(stream, a);
        return steps ? launch_serial<m40_bf16, true>(stream, a) : launch_serial<m40_bf16, false>(stream, a);
    }
    if (l->act_dtype != M40LLM_ACT_BF16 || !l->chunk_base || !l->chunks || l->n_chunks == 0 || !l->scratch || !m40_aligned16(l->scratch) ||
        l->scratch_bytes < m40llm_ext_lightning_scratch_bytes(l->n_chunks, l->heads, l->dim, l->vdim))
        return -4;
    a.steps = reinterpret_cast<float*>(static_cast<char*>(l->scratch) + state_bytes(l->n_chunks, l->heads, l->dim, l->vdim));
    return steps ? launch_chunked<true>(stream, a) : launch_chunked<false>(stream, a);
}

}  // extern "C"
