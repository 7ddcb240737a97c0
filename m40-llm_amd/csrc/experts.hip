// Choice of experts and the list of rows sorted by expert that the products per expert work through.  Everything is counted in a fixed
// order: no result depends on the order in which workgroups run.
#include "packed_gemm.hpp"

namespace {

constexpr uint32_t kThreads = 256, kWaves = kThreads / 64;
constexpr uint32_t kMost = M40LLM_MAX_EXPERTS, kPerLane = kMost / 64;
constexpr uint32_t kSmallPairs = 4096;     // (row, choice) pairs one workgroup keeps in LDS

// A wave routes one row: lane l holds experts l, l + 64, ...
__device__ __forceinline__ void route_row(const M40llmRoute& a, uint32_t row, uint32_t lane, uint32_t* ids, float* weight) {
    const uint32_t n = a.experts + a.identity;
    const float* z = static_cast<const float*>(a.logits) + (size_t)row * a.ld_logits;
    const float* correction = static_cast<const float*>(a.correction);
    float s[kPerLane], choice[kPerLane];
    float top = -INFINITY;
#pragma unroll
    for (uint32_t i = 0; i < kPerLane; ++i) {
        const uint32_t e = lane + 64u * i;
        s[i] = e < n ? z[e] : -INFINITY;
        top = fmaxf(top, s[i]);
    }
    top = m40_max64(top);
    float sum = 0.0f;
#pragma unroll
    for (uint32_t i = 0; i < kPerLane; ++i) {
        s[i] = lane + 64u * i < n ? expf(s[i] - top) : 0.0f;
        sum += s[i];
    }
    sum = m40_sum64(sum);
#pragma unroll
    for (uint32_t i = 0; i < kPerLane; ++i) {
        const uint32_t e = lane + 64u * i;
        s[i] /= sum;
        choice[i] = e < n ? s[i] + correction[e] : -INFINITY;
    }
    uint32_t taken = 0;                      // bit i: this lane's expert i is chosen
    for (uint32_t j = 0; j < a.top; ++j) {
        float best = -INFINITY;
        uint32_t at = 0xffffffffu;
#pragma unroll
        for (uint32_t i = 0; i < kPerLane; ++i) {
            const uint32_t e = lane + 64u * i;
            if (e < n && !(taken >> i & 1u) && (at == 0xffffffffu || choice[i] > best)) {
                best = choice[i];
                at = e;
            }
        }
#pragma unroll
        for (int d = 1; d < 64; d *= 2) {
            const float other = __shfl_xor(best, d);
            const uint32_t where = (uint32_t)__shfl_xor((int)at, d);
            const bool take = where != 0xffffffffu && (at == 0xffffffffu || other > best || (other == best && where < at));
            best = take ? other : best;
            at = take ? where : at;
        }
        float w = 0.0f;
#pragma unroll
        for (uint32_t i = 0; i < kPerLane; ++i)
            if (lane + 64u * i == at) {
                taken |= 1u << i;
                w = s[i];
            }
        if (at % 64u == lane) {
            ids[j] = at;
            weight[j] = w;
        }
    }
}

__global__ __launch_bounds__(kThreads) void route_rows_kernel(M40llmRoute a) {
    const uint32_t row = blockIdx.x * kWaves + (threadIdx.x >> 6);
    if (row >= a.rows) return;
    route_row(a, row, threadIdx.x & 63u, a.ids + (size_t)row * a.top, static_cast<float*>(a.weight) + (size_t)row * a.top);
}

// A workgroup an expert.  SMALL: it first routes all rows itself (one launch for a step of few rows).
template <bool SMALL>
__global__ __launch_bounds__(kThreads) void expert_lists_kernel(M40llmRoute a) {
    __shared__ uint32_t count[kMost];
    __shared__ uint32_t own_ids[SMALL ? kSmallPairs : 1];
    __shared__ float own_weight[SMALL ? kSmallPairs : 1];
    __shared__ uint32_t wave_n[kWaves], wave_slots[kWaves], wave_jobs[kWaves], wave_all[kWaves];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, mine = blockIdx.x, pairs = a.rows * a.top, E = a.experts;
    for (uint32_t e = tid; e < E; e += kThreads) count[e] = 0u;
    if (SMALL)
        for (uint32_t row = wave; row < a.rows; row += kWaves) route_row(a, row, lane, own_ids + row * a.top, own_weight + row * a.top);
    __syncthreads();
    const uint32_t* ids = SMALL ? own_ids : a.ids;
    for (uint32_t p = tid; p < pairs; p += kThreads) {
        const uint32_t e = ids[p];
        if (e < E) atomicAdd(&count[e], 1u);
        if (mine == 0u) {
            if (e >= E) a.place[p] = M40LLM_PLACE_INPUT;
            if (SMALL) {
                a.ids[p] = e;
                static_cast<float*>(a.weight)[p] = own_weight[p];
            }
        }
    }
    __syncthreads();
    // slots and jobs of the experts before this one, and all jobs
    uint32_t slots = 0, jobs = 0, all = 0;
    for (uint32_t e = tid; e < E; e += kThreads) {
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
    for (uint32_t w = 0; w < kWaves; ++w) { slots += wave_slots[w]; jobs += wave_jobs[w]; all += wave_all[w]; }
    if (mine == 0u && tid == 0u) a.jobs[0] = all;
    const uint32_t n = count[mine];
    for (uint32_t j = tid; j * a.job_rows < n; j += kThreads) {
        uint32_t* job = a.jobs + 4u + 4u * (jobs + j);
        const uint32_t left = n - j * a.job_rows;
        job[0] = mine;
        job[1] = slots + j * a.job_rows;
        job[2] = left < a.job_rows ? left : a.job_rows;
        job[3] = 0u;
    }
    if (n == 0u) return;
    // its rows in order
    uint32_t found = 0;
    for (uint32_t p0 = 0; p0 < pairs; p0 += kThreads) {
        const uint32_t p = p0 + tid;
        const bool hit = p < pairs && ids[p] == mine;
        const unsigned long long mask = __ballot(hit);
        if (lane == 0u) wave_n[wave] = (uint32_t)__popcll(mask);
        __syncthreads();
        uint32_t before = found;
#pragma unroll
        for (uint32_t w = 0; w < kWaves; ++w) {
            if (w < wave) before += wave_n[w];
            found += wave_n[w];
        }
        if (hit) {
            const uint32_t slot = slots + before + (uint32_t)__popcll(mask & ((1ull << lane) - 1ull));
            a.rows_of[slot] = p / a.top;
            a.place[p] = slot;
        }
        __syncthreads();
    }
    if (tid < ((n + 15u) & ~15u) - n) a.rows_of[slots + n + tid] = 0u;
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
    if (!ctx || !r || !r->logits || !r->correction || !r->ids || !r->weight || !r->rows_of || !r->place || !r->jobs) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    if (r->rows == 0 || r->experts == 0 || r->experts + r->identity > kMost || r->top == 0 || r->top > r->experts + r->identity ||
        r->ld_logits < r->experts + r->identity || (r->job_rows != 16u && r->job_rows != 32u && r->job_rows != 64u && r->job_rows != 128u) ||
        m40llm_ext_expert_slots(r->rows, r->experts, r->top) == 0 || m40llm_ext_expert_max_jobs(r->rows, r->experts, r->top, r->job_rows) == 0)
        return -3;
    (void)hipGetLastError();
    if (r->rows <= 64u && r->rows * r->top <= kSmallPairs) {
        expert_lists_kernel<true><<<r->experts, kThreads, 0, stream>>>(*r);
    } else {
        route_rows_kernel<<<(r->rows + kWaves - 1u) / kWaves, kThreads, 0, stream>>>(*r);
        expert_lists_kernel<false><<<r->experts, kThreads, 0, stream>>>(*r);
    }
    return hipGetLastError() == hipSuccess ? 0 : -2;
}

}  // extern "C"
