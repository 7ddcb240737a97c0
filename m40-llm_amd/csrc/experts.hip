// Choice of experts and the list of rows sorted by expert that the products per expert work through.  Everything is counted in a fixed
// order: no result depends on the order in which workgroups run.
#include "packed_gemm.hpp"

namespace {

constexpr uint32_t kThreads = 256, kWaves = kThreads / 64;
constexpr uint32_t kListThreads = 1024, kListWaves = kListThreads / 64;
constexpr uint32_t kMost = M40LLM_MAX_EXPERTS;
constexpr uint32_t kSmallPairs = 4096;     // (row, choice) pairs one workgroup keeps in LDS

// Experts in groups of `size` neighbours: what is left of `left` when only the `keep` groups whose best choice is largest (the lower group of
// equals) can be chosen from.
template <uint32_t N>
__device__ __forceinline__ uint32_t within_groups(const M40llmRoute& a, uint32_t lane, uint32_t size, const float (&choice)[N], uint32_t left) {
    uint32_t kept = 0, open = left;          // bit i: this lane's expert i is in a group that is taken, in one that still can be
    for (uint32_t k = 0; k < a.keep; ++k) {
        float best = -INFINITY;
#pragma unroll
        for (uint32_t i = 0; i < N; ++i) best = open >> i & 1u ? fmaxf(best, choice[i]) : best;
        best = m40_max64(best);
        uint32_t at = 0xffffffffu;           // its lowest expert (of one that is no number: the lowest that is open)
#pragma unroll
        for (uint32_t any = 0; any < 2u; ++any)
#pragma unroll
            for (uint32_t i = 0; i < N; ++i) {
                const unsigned long long hit = __ballot((open >> i & 1u) && (any || choice[i] == best));
                if (at == 0xffffffffu && hit) at = (uint32_t)__ffsll(hit) - 1u + 64u * i;
            }
        if (at == 0xffffffffu) break;
        const uint32_t group = at / size;
#pragma unroll
        for (uint32_t i = 0; i < N; ++i)
            if ((left >> i & 1u) && (lane + 64u * i) / size == group) {
                kept |= 1u << i;
                open &= ~(1u << i);
            }
    }
    return kept;
}

// A wave routes one row: lane l holds experts l, l + 64, ..., N of them.
template <uint32_t N>
__device__ __forceinline__ void route_row(const M40llmRoute& a, uint32_t row, uint32_t lane, uint32_t* ids, float* weight) {
    const uint32_t n = a.experts + a.identity;
    const float* z = static_cast<const float*>(a.logits) + (size_t)row * a.ld_logits;
    const float* correction = static_cast<const float*>(a.correction);
    const bool sigmoid = a.score == M40LLM_SCORE_SIGMOID;
    float s[N], choice[N];
    float top = -INFINITY;
#pragma unroll
    for (uint32_t i = 0; i < N; ++i) {
        const uint32_t e = lane + 64u * i;
        s[i] = e < n ? z[e] : -INFINITY;
        choice[i] = correction && e < n ? correction[e] : 0.0f;
        top = fmaxf(top, s[i]);
    }
    top = m40_max64(top);
    float sum = 0.0f;
#pragma unroll
    for (uint32_t i = 0; i < N; ++i) {
        const float logit = s[i];
        s[i] = lane + 64u * i >= n ? 0.0f : sigmoid ? m40_sigmoid(logit) : expf(logit - top);
        sum += s[i];
        // sigmoids of large logits are equal in f32 where the logits are not: without a correction the logits decide
        if (sigmoid) choice[i] = correction ? choice[i] + s[i] : logit;
    }
    sum = m40_sum64(sum);
    uint32_t left = 0;                       // bit i: this lane's expert i can be chosen
#pragma unroll
    for (uint32_t i = 0; i < N; ++i) {
        const uint32_t e = lane + 64u * i;
        if (!sigmoid) {
            s[i] /= sum;
            choice[i] += s[i];
        }
        if (e < n) left |= 1u << i;
    }
    if (a.groups > 1u) left = within_groups<N>(a, lane, n / a.groups, choice, left);
    uint32_t mine_id = 0;
    float mine_weight = 0.0f;                // choice `lane`
    for (uint32_t j = 0; j < a.top; ++j) {
        float best = -INFINITY;
#pragma unroll
        for (uint32_t i = 0; i < N; ++i) best = left >> i & 1u ? fmaxf(best, choice[i]) : best;
        best = m40_max64(best);
        uint32_t at = 0;
        float w = 0.0f;
        bool found = false;                  // the lowest index of equals: i before lane
#pragma unroll
        for (uint32_t i = 0; i < N; ++i) {
            const unsigned long long hit = __ballot((left >> i & 1u) && choice[i] == best);
            if (!found && hit) {
                const uint32_t l = (uint32_t)__ffsll(hit) - 1u;
                at = l + 64u * i;
                w = __shfl(s[i], (int)l);
                if (lane == l) left &= ~(1u << i);
                found = true;
            }
        }
        if (!found) {                        // nothing comparable is left (not a number): the lowest index that can be chosen
#pragma unroll
            for (uint32_t i = 0; i < N; ++i) {
                const unsigned long long hit = __ballot(left >> i & 1u);
                if (!found && hit) {
                    const uint32_t l = (uint32_t)__ffsll(hit) - 1u;
                    at = l + 64u * i;
                    w = __shfl(s[i], (int)l);
                    if (lane == l) left &= ~(1u << i);
                    found = true;
                }
            }
        }
        if (lane == (j & 63u)) { mine_id = at; mine_weight = w; }
        if ((j & 63u) == 63u || j + 1u == a.top) {
            const uint32_t first = j & ~63u;
            if (first + lane <= j) {
                ids[first + lane] = mine_id;
                weight[first + lane] = mine_weight * a.scale;
            }
        }
    }
}

template <uint32_t N>
__global__ __launch_bounds__(kThreads) void route_rows_kernel(M40llmRoute a) {
    const uint32_t row = blockIdx.x * kWaves + (threadIdx.x >> 6);
    if (row >= a.rows) return;
    route_row<N>(a, row, threadIdx.x & 63u, a.ids + (size_t)row * a.top, static_cast<float*>(a.weight) + (size_t)row * a.top);
}

// A workgroup an expert.  N > 0: it first routes all rows itself (one launch for a step of few rows).
template <uint32_t N>
__global__ __launch_bounds__(kListThreads) void expert_lists_kernel(M40llmRoute a) {
    constexpr bool SMALL = N > 0;
    __shared__ uint32_t count[kMost];
    __shared__ __align__(16) uint32_t own_ids[SMALL ? kSmallPairs : 4];
    __shared__ float own_weight[SMALL ? kSmallPairs : 1];
    __shared__ uint32_t wave_n[2][kListWaves], wave_slots[kListWaves], wave_jobs[kListWaves], wave_all[kListWaves];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, mine = blockIdx.x, pairs = a.rows * a.top, E = a.experts;
    for (uint32_t e = tid; e < E; e += kListThreads) count[e] = 0u;
    if constexpr (SMALL)
        for (uint32_t row = wave; row < a.rows; row += kListWaves) route_row<N>(a, row, lane, own_ids + row * a.top, own_weight + row * a.top);
    __syncthreads();
    const uint32_t* ids = SMALL ? own_ids : a.ids;
    auto load4 = [&](uint32_t p, uint32_t (&e)[4]) __attribute__((always_inline)) {
        if (p + 4u <= pairs) {
            const uint4 v = *reinterpret_cast<const uint4*>(ids + p);
            e[0] = v.x; e[1] = v.y; e[2] = v.z; e[3] = v.w;
        } else {
#pragma unroll
            for (uint32_t i = 0; i < 4u; ++i) e[i] = p + i < pairs ? ids[p + i] : 0xffffffffu;
        }
    };
    for (uint32_t p = tid * 4u; p < pairs; p += kListThreads * 4u) {
        uint32_t e[4];
        load4(p, e);
#pragma unroll
        for (uint32_t i = 0; i < 4u; ++i) {
            if (e[i] < E) atomicAdd(&count[e[i]], 1u);
            if (mine == 0u && p + i < pairs) {
                if (e[i] >= E) a.place[p + i] = M40LLM_PLACE_INPUT;
                if (SMALL) {
                    a.ids[p + i] = e[i];
                    static_cast<float*>(a.weight)[p + i] = own_weight[p + i];
                }
            }
        }
    }
    __syncthreads();
    // slots and jobs of the experts before this one, and all jobs
    uint32_t slots = 0, jobs = 0, all = 0;
    for (uint32_t e = tid; e < E; e += kListThreads) {
        const uint32_t c = count[e], j = (c + a.job_rows - 1u) / a.job_rows;
        all += j;
        if (e < mine) {
            slots += (c + 15u) & ~15u;
            jobs += j;
        }
    }
#pragma unroll
    for (int d = 1; d < 64; d *= 2) {
        slots += (uint32_t)__shfl_xor((int)slots, d);
        jobs += (uint32_t)__shfl_xor((int)jobs, d);
        all += (uint32_t)__shfl_xor((int)all, d);
    }
    if (lane == 0u) { wave_slots[wave] = slots; wave_jobs[wave] = jobs; wave_all[wave] = all; }
    __syncthreads();
    slots = jobs = all = 0u;
#pragma unroll
    for (uint32_t w = 0; w < kListWaves; ++w) { slots += wave_slots[w]; jobs += wave_jobs[w]; all += wave_all[w]; }
    const uint32_t n = count[mine];
    if (mine == 0u && tid == 0u) a.jobs[0] = all;
    if (mine == E - 1u && tid == 0u) a.jobs[1] = slots + ((n + 15u) & ~15u);
    for (uint32_t j = tid; j * a.job_rows < n; j += kListThreads) {
        uint32_t* job = a.jobs + 4u + 4u * (jobs + j);
        const uint32_t left = n - j * a.job_rows;
        job[0] = mine;
        job[1] = slots + j * a.job_rows;
        job[2] = left < a.job_rows ? left : a.job_rows;
        job[3] = 0u;
    }
    if (n == 0u) return;
    // its rows in order: four pairs a thread at a time
    uint32_t found = 0, phase = 0;
    for (uint32_t p0 = 0; p0 < pairs; p0 += kListThreads * 4u, phase ^= 1u) {
        const uint32_t p = p0 + tid * 4u;
        uint32_t e[4];
        load4(p, e);
        uint32_t before = 0, total = 0;      // hits of lower lanes, of the wave
#pragma unroll
        for (uint32_t i = 0; i < 4u; ++i) {
            const unsigned long long mask = __ballot(e[i] == mine);
            before += (uint32_t)__popcll(mask & ((1ull << lane) - 1ull));
            total += (uint32_t)__popcll(mask);
        }
        if (lane == 0u) wave_n[phase][wave] = total;
        __syncthreads();
        before += found;
#pragma unroll
        for (uint32_t w = 0; w < kListWaves; ++w) {
            const uint32_t k = wave_n[phase][w];
            if (w < wave) before += k;
            found += k;
        }
#pragma unroll
        for (uint32_t i = 0; i < 4u; ++i)
            if (e[i] == mine) {
                const uint32_t slot = slots + before++;
                a.rows_of[slot] = (p + i) / a.top;
                a.place[p + i] = slot;
                if (a.slot_weight) static_cast<float*>(a.slot_weight)[slot] = SMALL ? own_weight[SMALL ? p + i : 0] : static_cast<const float*>(a.weight)[p + i];
            }
    }
    if (tid < ((n + 15u) & ~15u) - n) {
        a.rows_of[slots + n + tid] = 0u;
        if (a.slot_weight) static_cast<float*>(a.slot_weight)[slots + n + tid] = 0.0f;
    }
}

// A wave moves 16 x 32 operand tiles: 16 rows of the list side by side.
__global__ __launch_bounds__(kThreads) void gather_rows_kernel(const uint16_t* __restrict__ src, uint32_t ld, const uint32_t* __restrict__ rows_of,
                                                               const uint32_t* __restrict__ jobs, uint16_t* __restrict__ dst) {
    const uint32_t slot0 = blockIdx.x * 16u, lane = threadIdx.x & 63u;
    if (slot0 >= jobs[1]) return;
    const uint16_t* from = src + (size_t)rows_of[slot0 + (lane & 15u)] * ld + (lane >> 4) * 8u;
    uint16_t* to = dst + (size_t)slot0 * ld + lane * 8u;
    for (uint32_t k = threadIdx.x >> 6; k < ld / 32u; k += kWaves)
        *reinterpret_cast<uint4*>(to + (size_t)k * kM40Tile) = *reinterpret_cast<const uint4*>(from + (size_t)k * 32u);
}

template <uint32_t N>
void launch_route(hipStream_t stream, const M40llmRoute& r) {
    if (r.rows <= 64u && r.rows * r.top <= kSmallPairs) {
        expert_lists_kernel<N><<<r.experts, kListThreads, 0, stream>>>(r);
    } else {
        route_rows_kernel<N><<<(r.rows + kWaves - 1u) / kWaves, kThreads, 0, stream>>>(r);
        expert_lists_kernel<0><<<r.experts, kListThreads, 0, stream>>>(r);
    }
}

}  // namespace

extern "C" {

uint32_t m40llm_ext_expert_slots(uint32_t rows, uint32_t experts, uint32_t top) {
    const uint64_t pairs = (uint64_t)rows * top, used = pairs < experts ? pairs : experts;
    const uint64_t n = (pairs + 15u * used + 15u) / 16u * 16u;
    return n > 0x7fffffffu ? 0u : (uint32_t)n;
}
uint32_t m40llm_ext_expert_max_jobs(uint32_t rows, uint32_t experts, uint32_t top, uint32_t job_rows) {
    if (job_rows == 0) return 0;
    const uint64_t pairs = (uint64_t)rows * top, used = pairs < experts ? pairs : experts;
    const uint64_t n = used + (pairs - used) / job_rows;      // every expert in use has one job that may not be full
    return n > 65535u ? 0u : (uint32_t)(n ? n : 1u);
}

int m40llm_ext_route_rows_async(M40llmCudaContext* ctx, const M40llmRoute* r, uint32_t stream_kind) {
    if (!ctx || !r || !r->logits || !r->ids || !r->weight || !r->rows_of || !r->place || !r->jobs) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    if (r->rows == 0 || r->experts == 0 || r->score > M40LLM_SCORE_SIGMOID || r->experts + r->identity > kMost || r->top == 0 || r->top > r->experts + r->identity ||
        r->ld_logits < r->experts + r->identity || (r->job_rows != 16u && r->job_rows != 32u && r->job_rows != 64u && r->job_rows != 128u) ||
        !m40_aligned16(r->ids) || m40llm_ext_expert_slots(r->rows, r->experts, r->top) == 0 || m40llm_ext_expert_max_jobs(r->rows, r->experts, r->top, r->job_rows) == 0)
        return -3;
    const uint32_t all = r->experts + r->identity;
    if (r->groups > 1u && (all % r->groups != 0 || r->keep == 0 || r->keep > r->groups || r->top > r->keep * (all / r->groups))) return -3;
    (void)hipGetLastError();
    if (all <= 64u) launch_route<1>(stream, *r);
    else if (all <= 128u) launch_route<2>(stream, *r);
    else if (all <= 256u) launch_route<4>(stream, *r);
    else launch_route<16>(stream, *r);
    return hipGetLastError() == hipSuccess ? 0 : -2;
}

int m40llm_ext_gather_rows_async(M40llmCudaContext* ctx, const void* d_src_bf16, uint32_t ld, const uint32_t* d_rows_of, const uint32_t* d_jobs,
                                 uint32_t max_slots, void* d_dst_bf16, uint32_t stream_kind) {
    if (!ctx || !d_src_bf16 || !d_rows_of || !d_jobs || !d_dst_bf16) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    if (ld == 0 || ld % 32u != 0 || max_slots == 0 || max_slots % 16u != 0 || !m40_aligned16(d_src_bf16) || !m40_aligned16(d_dst_bf16)) return -3;
    gather_rows_kernel<<<max_slots / 16u, kThreads, 0, stream>>>(static_cast<const uint16_t*>(d_src_bf16), ld, d_rows_of, d_jobs,
                                                                static_cast<uint16_t*>(d_dst_bf16));
    return hipGetLastError() == hipSuccess ? 0 : -2;
}

}  // extern "C"
