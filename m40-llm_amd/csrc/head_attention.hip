// Causal attention of long portions over keys and values that have been brought out of the cache's latents, head by head (the two
// page products of packed_gemm.hip write them): a workgroup of four waves owns 128 queries of one head, a wave 32 of them, and
// walks the sequence's pages of 64 tokens.  A page's operands -- keys, the rotated key part straight from the cache page, values --
// are in instruction order in memory and go into two LDS buffers, one page ahead.
//
// Products are formed transposed, S' = K Q' and O' = V' P': a lane holds the scores of one query (lane % 16) for keys 4 g + r of
// every 16, and the values are stored with a page's tokens in exactly that order, so the weights a lane computes are its operand of
// the second product, and maximum, sum and rescaling are one value a lane.  The maximum is a reference point that moves only when
// some score lies 8 (as a power of two) above it; it starts at the sink, whose weight is then 1 and counts once.
#include "packed_gemm.hpp"

namespace {

constexpr int kPage = M40LLM_PAGE_TOKENS;
constexpr int kQueries = 128;
constexpr float kLog2e = 1.4426950408889634f;

template <int DKT, int DVT>
__global__ __launch_bounds__(256, 2) void head_attention_kernel(M40llmHeadAttention a) {
    typedef __attribute__((address_space(3))) void* lds_dst_t;
    typedef const __attribute__((address_space(1))) void* global_src_t;
    extern __shared__ __align__(16) uint8_t lds[];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), g = lane >> 4, li = lane & 15;
    const int head = blockIdx.x, kp = (int)a.plain_tiles, kr = (int)a.rot_tiles, kt = kp + kr, vt = (int)a.v_tiles;
    const int page_bytes = (4 * kt + 2 * vt) * 1024;
    const uint32_t row0 = a.jobs[4 * blockIdx.y], count = a.jobs[4 * blockIdx.y + 1], first = a.jobs[4 * blockIdx.y + 2];   // pages[first ...]
    const uint32_t pages = a.row_pos[row0 + count - 1u] / kPage + 1u;
    const m40_bf16 *keys = static_cast<const m40_bf16*>(a.keys), *values = static_cast<const m40_bf16*>(a.values), *cache = static_cast<const m40_bf16*>(a.cache);
    auto issue = [&](int buf, uint32_t p, uint32_t page) __attribute__((always_inline)) {
        uint8_t* base = lds + buf * page_bytes;
        // wave w: the tiles of key group w, then its share of the value tiles
        const m40_bf16* k = keys + ((size_t)(first + p) * 4 + wave) * a.heads * kp * kM40Tile + (size_t)head * kp * kM40Tile + lane * 8;
        for (int i = 0; i < kp; ++i)
            __builtin_amdgcn_global_load_lds((global_src_t)(k + (size_t)i * kM40Tile), (lds_dst_t)(base + (wave * kt + i) * 1024), 16, 0, 0);
        const m40_bf16* r = cache + (((size_t)page * 4 + wave) * a.entry_tiles + (a.entry_tiles - kr)) * kM40Tile + lane * 8;
        for (int i = 0; i < kr; ++i)
            __builtin_amdgcn_global_load_lds((global_src_t)(r + (size_t)i * kM40Tile), (lds_dst_t)(base + (wave * kt + kp + i) * 1024), 16, 0, 0);
        const m40_bf16* v = values + ((size_t)(first + p) * a.heads + head) * vt * (2 * kM40Tile) + lane * 8;
        for (int i = wave; i < 2 * vt; i += 4)
            __builtin_amdgcn_global_load_lds((global_src_t)(v + (size_t)i * kM40Tile), (lds_dst_t)(base + (4 * kt + i) * 1024), 16, 0, 0);
    };
    issue(0, 0, a.pages[first]);
    uint32_t next_page = a.pages[first + (pages > 1u ? 1u : 0u)];
    m40_bf16x8 qf[2][DKT];
    uint32_t pos[2], row[2];
    bool live[2];
#pragma unroll
    for (int b = 0; b < 2; ++b) {
        const uint32_t i = (uint32_t)(wave * 32 + b * 16 + li);
        live[b] = i < count;
        row[b] = row0 + (live[b] ? i : count - 1u);
        pos[b] = a.row_pos[row[b]];
        const m40_bf16* q = static_cast<const m40_bf16*>(a.queries) + m40_packed_at(row[b], (uint32_t)(head * kt * 32), a.ld_queries >> 5) + g * 128;
#pragma unroll
        for (int k = 0; k < DKT; ++k) qf[b][k] = *reinterpret_cast<const m40_bf16x8*>(q + (size_t)(k < kt ? k : kt - 1) * kM40Tile);
    }
    // the wave's first and last positions: pages past the last are not worked on, pages up to the first need no compares
    const uint32_t i_first = (uint32_t)wave * 32u, i_last = i_first + 31u;
    const bool wave_live = i_first < count;
    const uint32_t pos_first = a.row_pos[row0 + (wave_live ? i_first : count - 1u)], pos_last = a.row_pos[row0 + (i_last < count ? i_last : count - 1u)];
    const float c = a.scale * kLog2e;
    float ref[2], sum[2];
    m40_float4 o[DVT][2];
#pragma unroll
    for (int b = 0; b < 2; ++b) {
        ref[b] = static_cast<const float*>(a.sink)[head] * kLog2e;
        sum[b] = g == 0 ? 1.0f : 0.0f;
    }
#pragma unroll
    for (int j = 0; j < DVT; ++j)
#pragma unroll
        for (int b = 0; b < 2; ++b) o[j][b] = m40_float4{0.f, 0.f, 0.f, 0.f};
    int buf = 0;
    for (uint32_t p = 0; p < pages; ++p, buf ^= 1) {
        m40_wait_and_meet<0>();                  // page p has landed, and nobody reads the other buffer any more
        if (p + 1u < pages) {
            issue(buf ^ 1, p + 1u, next_page);
            next_page = a.pages[first + (p + 2u < pages ? p + 2u : p + 1u)];
        }
        if (!wave_live || p * kPage > pos_last) continue;
        const uint8_t* base = lds + buf * page_bytes + lane * 16;
        m40_float4 s[4][2];
#pragma unroll
        for (int t = 0; t < 4; ++t)
#pragma unroll
            for (int b = 0; b < 2; ++b) s[t][b] = m40_float4{0.f, 0.f, 0.f, 0.f};
        __builtin_amdgcn_s_setprio(1);
#pragma unroll
        for (int k = 0; k < DKT; ++k)
            if (k < kt) {
#pragma unroll
                for (int t = 0; t < 4; ++t) {
                    const m40_bf16x8 kf = *reinterpret_cast<const m40_bf16x8*>(base + (t * kt + k) * 1024);
#pragma unroll
                    for (int b = 0; b < 2; ++b) s[t][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[b][k], s[t][b], 0, 0, 0);
                }
            }
        __builtin_amdgcn_s_setprio(0);
        const bool whole = p * kPage + kPage - 1u <= pos_first;
        m40_bf16x8 pf[2][2];
#pragma unroll
        for (int b = 0; b < 2; ++b) {
            float top = -INFINITY;
#pragma unroll
            for (int t = 0; t < 4; ++t)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    float x = s[t][b][r] * c;
                    if (!whole) x = p * kPage + t * 16 + 4 * g + r <= pos[b] ? x : -INFINITY;
                    s[t][b][r] = x;
                    top = fmaxf(top, x);
                }
            if (__any(top > ref[b] + 8.0f)) {
                top = fmaxf(top, __shfl_xor(top, 16));
                top = fmaxf(top, __shfl_xor(top, 32));
                const float to = fmaxf(ref[b], top), f = __builtin_amdgcn_exp2f(ref[b] - to);
                ref[b] = to;
                sum[b] *= f;
#pragma unroll
                for (int j = 0; j < DVT; ++j) o[j][b] *= f;
            }
#pragma unroll
            for (int t = 0; t < 4; ++t)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const float e = __builtin_amdgcn_exp2f(s[t][b][r] - ref[b]);
                    sum[b] += e;
                    pf[b][t >> 1][(t & 1) * 4 + r] = static_cast<m40_bf16>(e);
                }
        }
        __builtin_amdgcn_s_setprio(1);
#pragma unroll
        for (int j = 0; j < DVT; ++j)
            if (j < vt) {
#pragma unroll
                for (int h = 0; h < 2; ++h) {
                    const m40_bf16x8 vf = *reinterpret_cast<const m40_bf16x8*>(base + (4 * kt + j * 2 + h) * 1024);
#pragma unroll
                    for (int b = 0; b < 2; ++b) o[j][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[b][h], o[j][b], 0, 0, 0);
                }
            }
        __builtin_amdgcn_s_setprio(0);
    }
    __builtin_amdgcn_s_waitcnt(m40_vm_lgkm_wait(0));
    if (!wave_live) return;
#pragma unroll
    for (int b = 0; b < 2; ++b) {
        float l = sum[b];
        l += __shfl_xor(l, 16);
        l += __shfl_xor(l, 32);
        const float gate = static_cast<const float*>(a.gate)[(size_t)row[b] * a.ld_gate + head];
        const float f = m40_sigmoid(gate) / l;
        if (!live[b]) continue;
#pragma unroll
        for (int j = 0; j < DVT; ++j) {
            const int d = j * 16 + 4 * g;
            if (j < vt && d < (int)a.vdim)
                m40_store_packed<m40_bf16>(static_cast<m40_bf16*>(a.out), (int)row[b], head * (int)a.vdim + d, (long)a.ld_out, o[j][b] * f, (int)a.vdim - d,
                                           a.vdim % 4u == 0);
        }
    }
}

int lds_bytes(uint32_t k_tiles, uint32_t v_tiles) { return (int)(2u * (4u * k_tiles + 2u * v_tiles) * 1024u); }

template <int DKT, int DVT>
int launch(hipStream_t stream, const M40llmHeadAttention& a) {
    static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(head_attention_kernel<DKT, DVT>),
                                                       hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    if (attr != hipSuccess) return -2;
    head_attention_kernel<DKT, DVT><<<dim3(a.heads, a.n_jobs), 256, lds_bytes(a.plain_tiles + a.rot_tiles, a.v_tiles), stream>>>(a);
    return hipGetLastError() == hipSuccess ? 0 : -2;
}

}  // namespace

extern "C" {

int m40llm_ext_head_attention_serves(uint32_t k_tiles, uint32_t v_tiles) { return k_tiles >= 1u && k_tiles <= 8u && v_tiles >= 1u && v_tiles <= 8u; }

int m40llm_ext_head_attention_async(M40llmCudaContext* ctx, const M40llmHeadAttention* p, uint32_t stream_kind) {
    if (!ctx || !p || !p->queries || !p->keys || !p->values || !p->cache || !p->sink || !p->gate || !p->row_pos || !p->pages || !p->jobs || !p->out) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    const uint32_t kt = p->plain_tiles + p->rot_tiles;
    if (p->heads == 0 || p->n_jobs == 0 || p->n_jobs > 65535u || p->vdim == 0 || p->v_tiles != (p->vdim + 15u) / 16u || p->ld_queries % 32u != 0 ||
        p->ld_queries < p->heads * kt * 32u || p->ld_out % 32u != 0 || p->ld_out < p->heads * p->vdim || p->rot_tiles > p->entry_tiles ||
        !m40llm_ext_head_attention_serves(kt, p->v_tiles))
        return -3;
    (void)hipGetLastError();
    if (kt <= 3u && p->v_tiles <= 4u) return launch<3, 4>(stream, *p);
    if (kt <= 3u) return launch<3, 8>(stream, *p);
    if (kt <= 6u && p->v_tiles <= 4u) return launch<6, 4>(stream, *p);
    if (kt <= 6u) return launch<6, 8>(stream, *p);
    return launch<8, 8>(stream, *p);
}

}  // extern "C"
