// Causal attention of long portions over keys and values that have been brought out of the cache's latents, head by head (the two
// page products of packed_gemm.hip write them): a workgroup owns 128 (or 64) queries of one head, a wave 32 (16) of them, and
// walks the sequence's pages of 64 tokens.  A page's operands -- keys, the rotated key part straight from the cache page, values --
// are in instruction order in memory and go into two LDS buffers, one page ahead.  Where LDS holds four buffers the workgroup has
// two groups of four waves, one for the even and one for the odd pages, whose sums meet at the end: causal work differs between
// workgroups by the length of the sequence, and this halves the longest walk.
//
// Products are formed transposed, S' = K Q' and O' = V' P': a lane holds the scores of one query (lane % 16) for keys 4 g + r of
// every 16, and the values are stored with a page's tokens in exactly that order, so the weights a lane computes are its operand of
// the second product, and maximum, sum and rescaling are one value a lane.  The maximum is a reference point that moves only when
// some score lies 8 (as a power of two) above it; it starts at the sink, whose weight is then 1 and counts once.
#include "packed_gemm.hpp"

namespace {

constexpr int kPage = M40LLM_PAGE_TOKENS;
constexpr float kLog2e = 1.4426950408889634f;

// QB: 16-query blocks of a wave; GROUPS of four waves
template <int DKT, int DVT, int QB, int GROUPS>
__global__ __launch_bounds__(GROUPS * 256, 2) void head_attention_kernel(M40llmHeadAttention a) {
    typedef __attribute__((address_space(3))) void* lds_dst_t;
    typedef const __attribute__((address_space(1))) void* global_src_t;
    extern __shared__ __align__(16) uint8_t lds[];
    const int lane = threadIdx.x & 63, w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), g = lane >> 4, li = lane & 15;
    const int wave = w & 3, group = w >> 2;
    const int head = blockIdx.x, kp = (int)a.plain_tiles, kr = (int)a.rot_tiles, kt = kp + kr, vt = (int)a.v_tiles;
    const int page_bytes = (4 * kt + 2 * vt) * 1024;
    const uint32_t row0 = a.jobs[4 * blockIdx.y], count = a.jobs[4 * blockIdx.y + 1], first = a.jobs[4 * blockIdx.y + 2];   // pages[first ...]
    const uint32_t pages = a.row_pos[row0 + count - 1u] / kPage + 1u;
    const m40_bf16 *keys = static_cast<const m40_bf16*>(a.keys), *values = static_cast<const m40_bf16*>(a.values), *cache = static_cast<const m40_bf16*>(a.cache);
    auto issue = [&](int buf, uint32_t p, uint32_t page) __attribute__((always_inline)) {
        uint8_t* base = lds + (group * 2 + buf) * page_bytes;
        // wave w of a group: the tiles of key group w, then its share of the value tiles
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
    const uint32_t steps = (pages + GROUPS - 1u) / GROUPS, last = pages - 1u;
    auto page_of = [&](uint32_t step) { const uint32_t p = step * GROUPS + group; return p < last ? p : last; };    // past the end: the last again
    issue(0, page_of(0), a.pages[first + page_of(0)]);
    uint32_t next_page = a.pages[first + page_of(1)];
    m40_bf16x8 qf[QB][DKT];
    uint32_t pos[QB], row[QB];
    bool live[QB];
#pragma unroll
    for (int b = 0; b < QB; ++b) {
        const uint32_t i = (uint32_t)(wave * 16 * QB + b * 16 + li);
        live[b] = i < count;
        row[b] = row0 + (live[b] ? i : count - 1u);
        pos[b] = a.row_pos[row[b]];
        const m40_bf16* q = static_cast<const m40_bf16*>(a.queries) + m40_packed_at(row[b], (uint32_t)(head * kt * 32), a.ld_queries >> 5) + g * 128;
#pragma unroll
        for (int k = 0; k < DKT; ++k) qf[b][k] = *reinterpret_cast<const m40_bf16x8*>(q + (size_t)(k < kt ? k : kt - 1) * kM40Tile);
    }
    // the wave's first and last positions: pages past the last are not worked on, pages up to the first need no compares
    const uint32_t i_first = (uint32_t)wave * 16u * QB, i_last = i_first + 16u * QB - 1u;
    const bool wave_live = i_first < count;
    const uint32_t pos_first = a.row_pos[row0 + (wave_live ? i_first : count - 1u)], pos_last = a.row_pos[row0 + (i_last < count ? i_last : count - 1u)];
    const float c = a.scale * kLog2e;
    float ref[QB], sum[QB];
    m40_float4 o[DVT][QB];
#pragma unroll
    for (int b = 0; b < QB; ++b) {
        ref[b] = static_cast<const float*>(a.sink)[head] * kLog2e;
        sum[b] = g == 0 && group == 0 ? 1.0f : 0.0f;
    }
#pragma unroll
    for (int j = 0; j < DVT; ++j)
#pragma unroll
        for (int b = 0; b < QB; ++b) o[j][b] = m40_float4{0.f, 0.f, 0.f, 0.f};
    int buf = 0;
    for (uint32_t step = 0; step < steps; ++step, buf ^= 1) {
        m40_wait_and_meet<0>();                  // the step's pages have landed, and nobody reads the other buffers any more
        if (step + 1u < steps) {
            issue(buf ^ 1, page_of(step + 1u), next_page);
            next_page = a.pages[first + page_of(step + 2u)];
        }
        const uint32_t p = step * GROUPS + group;
        if (!wave_live || p > last || p * kPage > pos_last) continue;
        const uint8_t* base = lds + (group * 2 + buf) * page_bytes + lane * 16;
        m40_float4 s[4][QB];
#pragma unroll
        for (int t = 0; t < 4; ++t)
#pragma unroll
            for (int b = 0; b < QB; ++b) s[t][b] = m40_float4{0.f, 0.f, 0.f, 0.f};
        __builtin_amdgcn_s_setprio(1);
#pragma unroll
        for (int k = 0; k < DKT; ++k)
            if (k < kt) {
#pragma unroll
                for (int t = 0; t < 4; ++t) {
                    const m40_bf16x8 kf = *reinterpret_cast<const m40_bf16x8*>(base + (t * kt + k) * 1024);
#pragma unroll
                    for (int b = 0; b < QB; ++b) s[t][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[b][k], s[t][b], 0, 0, 0);
                }
            }
        __builtin_amdgcn_s_setprio(0);
        const bool whole = p * kPage + kPage - 1u <= pos_first;
        m40_bf16x8 pf[QB][2];
#pragma unroll
        for (int b = 0; b < QB; ++b) {
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
                    for (int b = 0; b < QB; ++b) o[j][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[b][h], o[j][b], 0, 0, 0);
                }
            }
        __builtin_amdgcn_s_setprio(0);
    }
    if constexpr (GROUPS == 2) {
        m40_wait_and_meet<0>();                  // every buffer is free
        constexpr int kFloats = QB * (2 + 4 * DVT);      // of a lane
        float* mine = reinterpret_cast<float*>(lds) + (size_t)wave * kFloats * 64 + lane;
        if (group == 1) {
#pragma unroll
            for (int b = 0; b < QB; ++b) {
                mine[(b * 2) * 64] = ref[b];
                mine[(b * 2 + 1) * 64] = sum[b];
#pragma unroll
                for (int j = 0; j < DVT; ++j)
#pragma unroll
                    for (int r = 0; r < 4; ++r) mine[(QB * 2 + (b * DVT + j) * 4 + r) * 64] = o[j][b][r];
            }
        }
        m40_wait_and_meet<63>();
        if (group == 1) return;
#pragma unroll
        for (int b = 0; b < QB; ++b) {
            const float other = mine[(b * 2) * 64], to = fmaxf(ref[b], other);
            const float f0 = __builtin_amdgcn_exp2f(ref[b] - to), f1 = __builtin_amdgcn_exp2f(other - to);
            sum[b] = sum[b] * f0 + mine[(b * 2 + 1) * 64] * f1;
#pragma unroll
            for (int j = 0; j < DVT; ++j)
#pragma unroll
                for (int r = 0; r < 4; ++r) o[j][b][r] = o[j][b][r] * f0 + mine[(QB * 2 + (b * DVT + j) * 4 + r) * 64] * f1;
        }
    } else {
        __builtin_amdgcn_s_waitcnt(m40_vm_lgkm_wait(0));
    }
    if (!wave_live) return;
#pragma unroll
    for (int b = 0; b < QB; ++b) {
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

constexpr int kLdsMax = 160 * 1024;
int lds_bytes(uint32_t k_tiles, uint32_t v_tiles, int groups) { return groups * 2 * (int)(4u * k_tiles + 2u * v_tiles) * 1024; }

template <int DKT, int DVT, int QB, int GROUPS>
int launch(hipStream_t stream, const M40llmHeadAttention& a) {
    static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(head_attention_kernel<DKT, DVT, QB, GROUPS>),
                                                       hipFuncAttributeMaxDynamicSharedMemorySize, kLdsMax);
    if (attr != hipSuccess) return -2;
    constexpr int join = GROUPS == 2 ? 4 * 64 * QB * (2 + 4 * DVT) * 4 : 0;
    const int pages = lds_bytes(a.plain_tiles + a.rot_tiles, a.v_tiles, GROUPS);
    head_attention_kernel<DKT, DVT, QB, GROUPS><<<dim3(a.heads, a.n_jobs), GROUPS * 256, pages > join ? pages : join, stream>>>(a);
    return hipGetLastError() == hipSuccess ? 0 : -2;
}
template <int DKT, int DVT>
int launch_any(hipStream_t stream, const M40llmHeadAttention& a, int num_cus) {
    // with enough workgroups the short ones fill in behind the long ones, and two independent groups a CU run better than one of eight waves
    if (lds_bytes(a.plain_tiles + a.rot_tiles, a.v_tiles, 2) <= kLdsMax && (uint64_t)a.heads * a.n_jobs <= 3ull * (uint32_t)num_cus)
        return a.job_rows == 64u ? launch<DKT, DVT, 1, 2>(stream, a) : launch<DKT, DVT, 2, 2>(stream, a);
    return a.job_rows == 64u ? launch<DKT, DVT, 1, 1>(stream, a) : launch<DKT, DVT, 2, 1>(stream, a);
}

}  // namespace

extern "C" {

int m40llm_ext_head_attention_serves(uint32_t k_tiles, uint32_t v_tiles) { return k_tiles >= 1u && k_tiles <= 8u && v_tiles >= 1u && v_tiles <= 8u; }

int m40llm_ext_head_attention_async(M40llmCudaContext* ctx, const M40llmHeadAttention* p, uint32_t stream_kind) {
    if (!ctx || !p || !p->queries || !p->keys || !p->values || !p->cache || !p->sink || !p->gate || !p->row_pos || !p->pages || !p->jobs || !p->out) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    const uint32_t kt = p->plain_tiles + p->rot_tiles;
    if ((p->job_rows != 64u && p->job_rows != 128u) || p->heads == 0 || p->n_jobs == 0 || p->n_jobs > 65535u || p->vdim == 0 || p->v_tiles != (p->vdim + 15u) / 16u || p->ld_queries % 32u != 0 ||
        p->ld_queries < p->heads * kt * 32u || p->ld_out % 32u != 0 || p->ld_out < p->heads * p->vdim || p->rot_tiles > p->entry_tiles ||
        !m40llm_ext_head_attention_serves(kt, p->v_tiles))
        return -3;
    (void)hipGetLastError();
    if (kt <= 3u && p->v_tiles <= 4u) return launch_any<3, 4>(stream, *p, ctx->num_cus);
    if (kt <= 3u) return launch_any<3, 8>(stream, *p, ctx->num_cus);
    if (kt <= 6u && p->v_tiles <= 4u) return launch_any<6, 4>(stream, *p, ctx->num_cus);
    if (kt <= 6u) return launch_any<6, 8>(stream, *p, ctx->num_cus);
    return launch_any<8, 8>(stream, *p, ctx->num_cus);
}

}  // extern "C"
