// Products of tile-packed activations with tile-packed bf16 weights (packed_gemm.hpp has the layout and the last steps).
//
// rows_packed_kernel   a workgroup owns one or two column tiles for up to 64 rows and its waves share out K: weights go
//                      straight from memory into the matrix instruction's operand registers, one contiguous kilobyte a
//                      load, each tile read once per 64 rows; the waves' sums meet in LDS.  Decode steps and short
//                      portions, and every product in f32.
// tile_packed_kernel   bf16, more rows: 128 x (128 or 256) tiles of C, both operands staged through LDS by direct
//                      global-to-LDS loads, five or six steps of 32 k deep with one barrier a step.  The buffers hold
//                      operands in instruction order, so LDS reads are contiguous kilobytes as well.
//
// Products per expert: both kernels take a list of jobs (expert, rows of the list sorted by expert) made on the device; the rows are
// gathered from plain rows (few rows, gate and up) or lie packed in list order.
#include "packed_gemm.hpp"

#include <type_traits>

namespace {

struct PackedArgs {
    const void* a;
    const m40_bf16* w;
    long lda, a_batch, w_batch;
    int n_tiles, k_tiles, rows;
    int k_stride;                  // k tiles from one row tile of the weights to the next
    int k_total;                   // k tiles of all batches together where the batches are parts of K (else 0)
    // operand rows that lie in cache pages: row tile t is group t % 4 of page pages[t / 4]
    const uint32_t* pages;
    int page_k_tiles;
    const uint32_t *jobs, *gather; // products per expert
    int segment;                   // column tiles that read the same columns of a (0 = all): the next ones read those a_batch further
    __device__ int k_count(int batch) const { return k_total && k_total - batch * k_tiles < k_tiles ? k_total - batch * k_tiles : k_tiles; }
};

enum { kAllRows = 0, kJobSlots = 1, kJobGather = 2 };

template <class T, int MT, int NT, int WAVES, int JOBS>
__global__ __launch_bounds__(WAVES * 64) void rows_packed_kernel(PackedArgs g, M40Epilogue<T> e) {
    extern __shared__ __align__(16) float red[];       // [WAVES][MT][NT][64][4]
    typedef typename M40Act<T>::vec8 vec8;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int tile0 = (int)blockIdx.x * NT;
    int row0 = (int)blockIdx.y * 16 * MT, batch = blockIdx.z;
    if (JOBS != kAllRows) {
        if (blockIdx.y >= g.jobs[0]) return;
        const uint32_t* job = g.jobs + 4 + 4 * blockIdx.y;
        batch = (int)job[0];
        row0 = (int)job[1];
        g.rows = e.rows = row0 + (int)job[2];
    }
    constexpr long kStep = JOBS == kJobGather ? 32 : kM40Tile;       // elements from k tile to k tile
    const T* a[MT];
#pragma unroll
    for (int m = 0; m < MT; ++m) {
        const int rt = row0 / 16 + m, last = (g.rows - 1) / 16, c = rt < last ? rt : last;
        if (JOBS == kJobGather) a[m] = static_cast<const T*>(g.a) + (long)g.gather[c * 16 + (lane & 15)] * g.lda + (lane >> 4) * 8;
        else a[m] = static_cast<const T*>(g.a) + (JOBS == kAllRows ? (g.segment ? tile0 / g.segment : batch) * g.a_batch : 0) + (long)c * 16 * g.lda + lane * 8;
    }
    const m40_bf16* w[NT];
#pragma unroll
    for (int n = 0; n < NT; ++n) {
        const int t = tile0 + n < g.n_tiles ? tile0 + n : g.n_tiles - 1;
        w[n] = g.w + batch * g.w_batch + (long)t * g.k_stride * kM40Tile + lane * 8;
    }
    const int k_tiles = g.k_count(batch);
    m40_float4 acc[MT][NT];
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int n = 0; n < NT; ++n) acc[m][n] = m40_float4{0.f, 0.f, 0.f, 0.f};
    constexpr int U = sizeof(T) == 2 ? (MT * NT <= 2 ? 8 : 4) : 1;
    int k = wave;
    for (; k + (U - 1) * WAVES < k_tiles; k += U * WAVES) {
        uint4 wf[U][NT];
        vec8 af[U][MT];
#pragma unroll
        for (int u = 0; u < U; ++u)
#pragma unroll
            for (int n = 0; n < NT; ++n) wf[u][n] = m40_load_stream(reinterpret_cast<const uint4*>(w[n] + (long)(k + u * WAVES) * kM40Tile));
#pragma unroll
        for (int u = 0; u < U; ++u)
#pragma unroll
            for (int m = 0; m < MT; ++m) af[u][m] = M40Act<T>::load8(a[m] + (long)(k + u * WAVES) * kStep);
#pragma unroll
        for (int u = 0; u < U; ++u)
#pragma unroll
            for (int m = 0; m < MT; ++m)
#pragma unroll
                for (int n = 0; n < NT; ++n) acc[m][n] = M40Act<T>::mma(__builtin_bit_cast(m40_bf16x8, wf[u][n]), af[u][m], acc[m][n]);
    }
    for (; k < k_tiles; k += WAVES) {
        uint4 wf[NT];
#pragma unroll
        for (int n = 0; n < NT; ++n) wf[n] = *reinterpret_cast<const uint4*>(w[n] + (long)k * kM40Tile);
#pragma unroll
        for (int m = 0; m < MT; ++m) {
            const vec8 af = M40Act<T>::load8(a[m] + (long)k * kStep);
#pragma unroll
            for (int n = 0; n < NT; ++n) acc[m][n] = M40Act<T>::mma(__builtin_bit_cast(m40_bf16x8, wf[n]), af, acc[m][n]);
        }
    }
    m40_float4* r4 = reinterpret_cast<m40_float4*>(red);
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int n = 0; n < NT; ++n) r4[((wave * MT + m) * NT + n) * 64 + lane] = acc[m][n];
    __syncthreads();
    for (int m = wave; m < MT; m += WAVES) {
        if (row0 + m * 16 >= g.rows) continue;
        m40_float4 s[NT];
#pragma unroll
        for (int n = 0; n < NT; ++n) {
            s[n] = r4[(m * NT + n) * 64 + lane];
#pragma unroll
            for (int i = 1; i < WAVES; ++i) s[n] += r4[((i * MT + m) * NT + n) * 64 + lane];
        }
        if (NT == 2 && e.kind == M40LLM_PACKED_PROJECT && tile0 >= e.plain_tiles) {
            m40_epilogue_pair(e, row0 + m * 16, (tile0 - e.plain_tiles) / 2, lane, s[0], s[NT - 1]);
        } else {
#pragma unroll
            for (int n = 0; n < NT; ++n)
                if (tile0 + n < g.n_tiles) m40_epilogue_tile(e, JOBS == kAllRows ? batch : 0, row0 + m * 16, tile0 + n, lane, s[n]);
        }
    }
}

template <class T, int MT, int NT, int WAVES, int JOBS>
int launch_rows(hipStream_t stream, const PackedArgs& g, const M40Epilogue<T>& e, int batches) {
    // g.rows: with jobs, the most jobs there can be
    const dim3 grid((unsigned)((g.n_tiles + NT - 1) / NT), (unsigned)(JOBS == kAllRows ? (g.rows + 16 * MT - 1) / (16 * MT) : g.rows), (unsigned)batches);
    constexpr size_t lds = (size_t)WAVES * MT * NT * 1024;
    static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(rows_packed_kernel<T, MT, NT, WAVES, JOBS>),
                                                       hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (attr != hipSuccess) return -2;
    rows_packed_kernel<T, MT, NT, WAVES, JOBS><<<grid, WAVES * 64, lds, stream>>>(g, e);
    return hipGetLastError() == hipSuccess ? 0 : -2;
}

template <class T, int MT, int JOBS>
int launch_rows_m(hipStream_t stream, const PackedArgs& g, const M40Epilogue<T>& e, int batches) {
    if constexpr (JOBS != kJobSlots)
        if (e.kind == M40LLM_PACKED_PROJECT) return launch_rows<T, MT, 2, 8, JOBS>(stream, g, e, batches);
    if constexpr (JOBS != kJobGather) {
        if (g.k_tiles >= 64) return launch_rows<T, MT, 1, 16, JOBS>(stream, g, e, batches);
        if (g.k_tiles >= 16) return launch_rows<T, MT, 1, 8, JOBS>(stream, g, e, batches);
        return launch_rows<T, MT, 1, 4, JOBS>(stream, g, e, batches);
    }
    return -3;
}
template <class T, int JOBS>
int launch_rows_any(hipStream_t stream, const PackedArgs& g, const M40Epilogue<T>& e, int batches, int rows) {
    if (rows <= 16) return launch_rows_m<T, 1, JOBS>(stream, g, e, batches);
    if (rows <= 32) return launch_rows_m<T, 2, JOBS>(stream, g, e, batches);
    return launch_rows_m<T, 4, JOBS>(stream, g, e, batches);
}

// ---- many rows, bf16 ---------------------------------------------------------------------------------------------------
// Workgroup of four waves (2 x 2), wave tile 64 x (16 NTW): C tile 128 x 32 NTW.  A step is one k tile of every operand
// tile: (8 + 2 NTW) KB, filled by global_load_lds (a wave's instruction moves one 16 x 32 operand tile, a contiguous kilobyte).
//
// Memory instructions are issued under matrix instructions: the fragments of the next step and the loads of a step kBufs - 1
// ahead go out one at a time between the current step's products (sched_group_barrier), so that no wave waits for an address
// or LDS unit with the matrix pipe idle.  Step t refills the buffer of step t - 1, whose fragments every wave had in registers
// before the barrier behind that step, and ends with step t + 2 landed.
enum { kPlainRows = 0, kPageKeys = 1, kPageValues = 2, kSlots = 3 };
constexpr int tile_bufs(int ntw) { return ntw == 8 ? 6 : 5; }       // one or two workgroups a CU

template <int NTW, int FORM>
__global__ __launch_bounds__(256, 1) void tile_packed_kernel(PackedArgs g, M40Epilogue<m40_bf16> e) {
    typedef __attribute__((address_space(3))) void* lds_dst_t;
    typedef const __attribute__((address_space(1))) void* global_src_t;
    extern __shared__ __align__(16) uint8_t stage_lds[];
    constexpr int kATiles = 8, kBTiles = 2 * NTW;                    // 16-row operand tiles of the workgroup
    constexpr int kBufs = tile_bufs(NTW), kStepBytes = (kATiles + kBTiles) * 1024;
    constexpr int kLoads = (kATiles + kBTiles) / 4;                  // per wave and step
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    constexpr bool kJobs = FORM == kSlots;
    const int tiles_n = (g.n_tiles + kBTiles - 1) / kBTiles, tiles_m = kJobs ? (int)g.jobs[0] : (g.rows + 127) / 128;
    const int workgroups = kJobs ? tiles_m * tiles_n : (int)gridDim.x;       // the grid is as large as the list of jobs can be
    if (kJobs && (int)blockIdx.x >= workgroups) return;
    // workgroups are dealt to the eight dies in turn: each die gets a contiguous band of tiles, walked in blocks of four row
    // tiles so that what runs on a die at one time shares both operands
    const int per_die = workgroups / 8;
    const int logical = (int)blockIdx.x < per_die * 8 ? ((int)blockIdx.x % 8) * per_die + (int)blockIdx.x / 8 : (int)blockIdx.x;
    const int group = logical / (4 * tiles_n), in_group = logical - group * 4 * tiles_n, gm = tiles_m - group * 4 < 4 ? tiles_m - group * 4 : 4;
    const int t0 = in_group / gm * kBTiles;
    int m0 = (group * 4 + in_group % gm) * 128, batch = blockIdx.z;
    if (kJobs) {
        const uint32_t* job = g.jobs + 4 + 4 * (group * 4 + in_group % gm);
        batch = __builtin_amdgcn_readfirstlane((int)job[0]);
        m0 = __builtin_amdgcn_readfirstlane((int)job[1]);
        g.rows = e.rows = m0 + __builtin_amdgcn_readfirstlane((int)job[2]);
    }
    const m40_bf16* A = static_cast<const m40_bf16*>(g.a) + (kJobs ? 0 : (g.segment ? t0 / g.segment : batch) * g.a_batch);
    const m40_bf16* W = g.w + batch * g.w_batch;
    const int k_tiles = g.k_count(batch);
    // this wave's pieces of a step: operand tiles wave, wave + 4, ... of the A tiles, then of the W tiles
    const m40_bf16* src[kLoads];
#pragma unroll
    for (int i = 0; i < kLoads; ++i) {
        const int t = wave + 4 * i;
        if (i < kATiles / 4) {
            if (FORM == kPageKeys || FORM == kPageValues) {
                const int rt = m0 / 16 + t, tiles = g.rows / 16, c = rt < tiles ? rt : tiles - 1;
                src[i] = A + ((long)g.pages[c >> 2] * 4 + (c & 3)) * g.page_k_tiles * kM40Tile + lane * 8;
            } else {
                const int rt = m0 / 16 + t, last = (g.rows - 1) / 16;
                src[i] = A + (long)(rt < last ? rt : last) * 16 * g.lda + lane * 8;
            }
        } else {
            const int n = t0 + t - kATiles;
            src[i] = W + (long)(n < g.n_tiles ? n : g.n_tiles - 1) * g.k_stride * kM40Tile + lane * 8;
        }
    }
    auto issue = [&](int buf, int t) __attribute__((always_inline)) {
        uint8_t* base = stage_lds + buf * kStepBytes + wave * 1024;
        const int k = t < k_tiles ? t : k_tiles - 1;                 // past the end: loaded again, not used
#pragma unroll
        for (int i = 0; i < kLoads; ++i)
            __builtin_amdgcn_global_load_lds((global_src_t)(src[i] + (long)k * kM40Tile), (lds_dst_t)(base + i * 4096), 16, 0, 0);
    };
    const int wm = wave >> 1, wn = wave & 1;
    m40_float4 acc[4][NTW];
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < NTW; ++j) acc[i][j] = m40_float4{0.f, 0.f, 0.f, 0.f};
    struct Frags { m40_bf16x8 a[4], b[NTW]; } f[2];
    auto read_frags = [&](Frags& f, int buf) __attribute__((always_inline)) {
        const uint8_t* a = stage_lds + buf * kStepBytes + wm * 4096 + lane * 16;
        const uint8_t* b = stage_lds + buf * kStepBytes + (kATiles + wn * NTW) * 1024 + lane * 16;
#pragma unroll
        for (int i = 0; i < 4; ++i) f.a[i] = *reinterpret_cast<const m40_bf16x8*>(a + i * 1024);
#pragma unroll
        for (int j = 0; j < NTW; ++j) f.b[j] = *reinterpret_cast<const m40_bf16x8*>(b + j * 1024);
    };
    auto compute = [&](const Frags& f) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
            for (int j = 0; j < NTW; ++j)
                acc[i][j] = FORM == kPageValues ? __builtin_amdgcn_mfma_f32_16x16x32_bf16(f.a[i], f.b[j], acc[i][j], 0, 0, 0)
                                                : __builtin_amdgcn_mfma_f32_16x16x32_bf16(f.b[j], f.a[i], acc[i][j], 0, 0, 0);
    };
#pragma unroll
    for (int i = 0; i < kBufs - 1; ++i) issue(i, i);
    m40_wait_and_meet<(kBufs - 3) * kLoads>();                       // steps 0 and 1 have landed
    read_frags(f[0], 0);
    int buf = 0;
    auto step = [&](auto parity, int t) __attribute__((always_inline)) {
        constexpr int ph = decltype(parity)::value;
        const int next = buf == kBufs - 1 ? 0 : buf + 1;
        read_frags(f[ph ^ 1], next);
        issue(buf == 0 ? kBufs - 1 : buf - 1, t + kBufs - 1);
        compute(f[ph]);
        // products between two fragment reads, and between two loads
        constexpr int kPerRead = NTW == 8 ? 2 : 1, kPerLoad = (4 * NTW - kPerRead * (4 + NTW)) / kLoads;
#pragma unroll
        for (int i = 0; i < 4 + NTW; ++i) {
            __builtin_amdgcn_sched_group_barrier(0x008, kPerRead, 0);
            __builtin_amdgcn_sched_group_barrier(0x100, 1, 0);
        }
#pragma unroll
        for (int i = 0; i < kLoads; ++i) {
            __builtin_amdgcn_sched_group_barrier(0x008, kPerLoad, 0);
            __builtin_amdgcn_sched_group_barrier(0x020, 1, 0);
        }
        m40_wait_and_meet<(kBufs - 3) * kLoads>();
        buf = next;
    };
    int t = 0;
    for (; t + 2 <= k_tiles; t += 2) {
        step(std::integral_constant<int, 0>(), t);
        step(std::integral_constant<int, 1>(), t + 1);
    }
    if (t < k_tiles) compute(f[0]);
    m40_wait_and_meet<0>();                                          // every load has landed: the buffers are free
    // The sums go through LDS (each wave its own) so that the last step is a loop of a few instructions and not 4 NTW copies of it:
    // run once per workgroup, those would be fetched cold.
    m40_float4* mine = reinterpret_cast<m40_float4*>(stage_lds) + wave * 4 * NTW * 64 + lane;
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < NTW; ++j) mine[(i * NTW + j) * 64] = acc[i][j];
    if (FORM == kPlainRows && e.kind == M40LLM_PACKED_ADD && e.vec_out && e.cols % 16 == 0) {
        // the old values of four tiles are requested together, under clamped addresses: loads behind a branch would be awaited one by one
#pragma unroll 1
        for (int i = 0; i < NTW; ++i) {
            const int row = m0 + (wm * 4 + i * 4 / NTW) * 16 + (lane & 15), j0 = i * 4 % NTW;
            float* o = e.out_f32 + batch * e.out_batch + (long)(row < e.rows ? row : e.rows - 1) * e.ld_out + 4 * (lane >> 4);
            m40_float4 old[4];
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int col = (t0 + wn * NTW + j0 + j) * 16;
                old[j] = *reinterpret_cast<const m40_float4*>(o + (col < e.cols ? col : 0));
            }
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int col = (t0 + wn * NTW + j0 + j) * 16;
                if (row < e.rows && col < e.cols) *reinterpret_cast<m40_float4*>(o + col) = old[j] + mine[(i * 4 + j) * 64];
            }
        }
        return;
    }
#pragma unroll 1
    for (int p = 0; p < 2 * NTW; ++p) {
        const int i = p / (NTW / 2), j = p % (NTW / 2) * 2, row0 = m0 + (wm * 4 + i) * 16, tile = t0 + wn * NTW + j;
        if (row0 >= g.rows || tile >= g.n_tiles) continue;
        const m40_float4 v0 = mine[(2 * p) * 64], v1 = mine[(2 * p + 1) * 64];
        const bool second = tile + 1 < g.n_tiles;
        if (FORM == kPageValues) {
            m40_epilogue_values(e, row0, tile, lane, v0);
            if (second) m40_epilogue_values(e, row0, tile + 1, lane, v1);
        } else if (e.kind == M40LLM_PACKED_PROJECT && tile >= e.plain_tiles) {
            if (second) m40_epilogue_pair(e, row0, (tile - e.plain_tiles) / 2, lane, v0, v1);
        } else {
#pragma unroll 1
            for (int k = 0; k < (second ? 2 : 1); ++k) m40_epilogue_tile(e, kJobs ? 0 : batch, row0, tile + k, lane, k ? v1 : v0);
        }
    }
}

template <int NTW, int FORM>
int launch_tile(hipStream_t stream, const PackedArgs& g, const M40Epilogue<m40_bf16>& e, int batches) {
    constexpr int lds = (8 + 2 * NTW) * 1024 * tile_bufs(NTW);
    static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(tile_packed_kernel<NTW, FORM>),
                                                       hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    if (attr != hipSuccess) return -2;
    constexpr bool kJobs = FORM == kSlots;        // g.rows: the most jobs there can be
    const long long tiles = (long long)(kJobs ? g.rows : (g.rows + 127) / 128) * ((g.n_tiles + 2 * NTW - 1) / (2 * NTW));
    tile_packed_kernel<NTW, FORM><<<dim3((unsigned)tiles, 1, (unsigned)batches), 256, lds, stream>>>(g, e);
    return hipGetLastError() == hipSuccess ? 0 : -2;
}
template <int FORM>
int launch_tile_any(hipStream_t stream, const PackedArgs& g, const M40Epilogue<m40_bf16>& e, int batches, int num_cus) {
    const long long wide = (long long)(FORM == kSlots ? g.rows : (g.rows + 127) / 128) * ((g.n_tiles + 15) / 16) * batches;
    // a short sum is mostly a workgroup's start and end: two narrower workgroups a CU cover each other's
    if (wide * 16 >= 9ll * num_cus && g.k_tiles > (FORM == kSlots && e.kind == M40LLM_PACKED_STORE_ACT ? 64 : 32)) return launch_tile<8, FORM>(stream, g, e, batches);
    return launch_tile<4, FORM>(stream, g, e, batches);
}

template <class T>
M40Epilogue<T> make_epilogue(const M40llmPackedGemm& p) {
    M40Epilogue<T> e{};
    e.kind = (int)p.epilogue;
    e.rows = (int)p.rows;
    e.out_f32 = static_cast<float*>(p.out_f32);
    e.out_act = static_cast<T*>(p.out_act);
    e.ld_out = (long)p.ld_out; e.ld_act = (long)p.ld_act;
    e.out_batch = (long)p.out_batch; e.act_batch = (long)p.act_batch;
    e.cols = (int)p.cols;
    auto aligned = [](const void* q, size_t n) { return reinterpret_cast<uintptr_t>(q) % n == 0; };
    e.vec_out = p.ld_out % 4 == 0 && p.out_batch % 4 == 0 && aligned(p.out_f32, 16);
    e.vec_act = p.ld_act % 4 == 0 && p.act_batch % 4 == 0 && aligned(p.out_act, 4 * sizeof(T));
    e.plain_tiles = (int)p.plain_tiles;
    e.activation = (int)p.activation;
    e.act_alpha = p.act_alpha; e.act_limit = p.act_limit;
    e.row_scale = static_cast<const float*>(p.row_scale);
    e.out_scale = p.out_scale; e.out_cap = p.out_cap;
    e.n_tiles = (int)p.n_tiles; e.act_col = (int)p.act_col;
    e.gate = static_cast<const float*>(p.gate);
    e.ld_gate = (long)p.ld_gate;
    e.head_width = (int)p.head_width; e.rot_start = (int)p.rot_start; e.heads = (int)p.heads;
    e.split_row = (int)p.split_row; e.rot_half = (int)p.rot_half;
    e.angles = static_cast<const float2*>(p.angles);
    e.rot_out = static_cast<T*>(p.rot_out);
    e.ld_rot = (long)p.ld_rot;
    return e;
}

// one thread per source element
__global__ __launch_bounds__(256) void pack_tiles_kernel(const uint16_t* __restrict__ src, uint16_t* __restrict__ dst,
                                                         M40llmPackPlan p, size_t total) {
    for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < total; i += (size_t)gridDim.x * 256) {
        size_t r = i;
        const uint32_t k = (uint32_t)(r % p.k); r /= p.k;
        const uint32_t kb = (uint32_t)(r % p.k_blocks); r /= p.k_blocks;
        const uint32_t n = (uint32_t)(r % p.n), nb = (uint32_t)(r / p.n);
        const uint32_t row = p.n_offset + nb * p.n_block_pad + n, col = p.k_offset + kb * p.k_block_pad + k;
        const size_t tile = (size_t)(p.tile_first + (row >> 4) * p.tile_stride) * p.k_tiles + (col >> 5);
        dst[tile * kM40Tile + m40_tile_offset(row & 15u, col & 31u)] = src[nb * p.sn_block + n * p.sn + kb * p.sk_block + k * p.sk];
    }
}

__global__ __launch_bounds__(256) void clear_u32_kernel(uint32_t* dst, size_t n) {
    for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (size_t)gridDim.x * 256) dst[i] = 0u;
}

__global__ __launch_bounds__(256) void fill_random_bf16_kernel(uint16_t* dst, size_t n, uint64_t seed, float half_range) {
    for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (size_t)gridDim.x * 256) {
        uint64_t z = seed + (i + 1) * 0x9e3779b97f4a7c15ull;        // splitmix64
        z = (z ^ (z >> 30)) * 0xbf58476d1ce4e5b9ull;
        z = (z ^ (z >> 27)) * 0x94d049bb133111ebull;
        z ^= z >> 31;
        const float u = (float)(uint32_t)(z >> 40) * (2.0f / 16777216.0f) - 1.0f;
        dst[i] = __builtin_bit_cast(uint16_t, static_cast<m40_bf16>(u * half_range));
    }
}

}  // namespace

extern "C" {

int m40llm_ext_fill_random_bf16_async(M40llmCudaContext* ctx, void* d_dst, uint64_t n, uint64_t seed, float std_dev, uint32_t stream_kind) {
    if (!ctx || !d_dst) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    if (n == 0) return 0;
    const uint64_t blocks = (n + 255) / 256;
    fill_random_bf16_kernel<<<(unsigned)(blocks < 65536 ? blocks : 65536), 256, 0, stream>>>(static_cast<uint16_t*>(d_dst), (size_t)n, seed,
                                                                                             std_dev * 1.7320508075688772f);
    return hipGetLastError() == hipSuccess ? 0 : -2;
}

int m40llm_ext_pack_tiles_async(M40llmCudaContext* ctx, const void* d_src, void* d_dst, const M40llmPackPlan* plan, uint32_t stream_kind) {
    if (!ctx || !d_src || !d_dst || !plan) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    const M40llmPackPlan& p = *plan;
    const size_t total = (size_t)p.n_blocks * p.n * p.k_blocks * p.k;
    if (total == 0 || p.tile_stride == 0) return -3;
    if (p.k_offset + (uint64_t)(p.k_blocks - 1) * p.k_block_pad + p.k > (uint64_t)p.k_tiles * 32u) return -3;
    const size_t blocks = (total + 255) / 256;
    pack_tiles_kernel<<<(unsigned)(blocks < 65536 ? blocks : 65536), 256, 0, stream>>>(static_cast<const uint16_t*>(d_src),
                                                                                       static_cast<uint16_t*>(d_dst), p, total);
    return hipGetLastError() == hipSuccess ? 0 : -2;
}

int m40llm_ext_clear_u32_async(M40llmCudaContext* ctx, void* d_dst, size_t n, uint32_t stream_kind) {
    if (!ctx || !d_dst) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    if (n == 0) return 0;
    const size_t blocks = (n + 255) / 256;
    clear_u32_kernel<<<(unsigned)(blocks < 4096 ? blocks : 4096), 256, 0, stream>>>(static_cast<uint32_t*>(d_dst), n);
    return hipGetLastError() == hipSuccess ? 0 : -2;
}

int m40llm_ext_packed_gemm_async(M40llmCudaContext* ctx, const M40llmPackedGemm* p, uint32_t stream_kind) {
    if (!ctx || !p || !p->a || !p->w) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    const bool paged = p->epilogue == M40LLM_PACKED_KEYS || p->epilogue == M40LLM_PACKED_VALUES;
    const uint32_t k_parts = p->k_parts > 1u ? p->k_parts : 1u, part_tiles = (p->k_tiles + k_parts - 1) / k_parts;
    if (p->act_dtype > 1u || p->epilogue > M40LLM_PACKED_CAP || p->activation > M40LLM_LIMITED_GATE || p->rows == 0 || p->batches == 0 || p->batches > 65535u ||
        p->n_tiles == 0 || p->k_tiles == 0 || !m40_aligned16(p->a) || !m40_aligned16(p->w) || p->rows > 0x3fffffffu ||
        (p->batches > 1u && (p->a_batch % 32 != 0 || p->w_batch % 8 != 0)))
        return -3;
    if (p->jobs && (p->batches != 1u || k_parts > 1u || p->max_jobs == 0 || p->max_jobs > 65535u || (p->job_rows != 16u && p->job_rows != 32u && p->job_rows != 64u && p->job_rows != 128u) ||
                    (p->job_rows == 128u && p->act_dtype == M40LLM_ACT_F32) || p->w_batch % 8 != 0 ||
                    !(p->epilogue == M40LLM_PACKED_STORE_ACT ? !p->gather
                                                                  : p->epilogue == M40LLM_PACKED_PROJECT && p->plain_tiles == 0 && (p->job_rows == 128u) == !p->gather)))
        return -3;
    if (!paged && (p->lda % 32 != 0 || p->lda < (uint64_t)p->k_tiles * 32u)) return -3;
    // a workgroup's column tiles lie in one segment
    if (p->segment_tiles && (paged || p->jobs || p->batches != 1u || k_parts > 1u || p->epilogue == M40LLM_PACKED_PROJECT || p->segment_tiles % 16u != 0 || p->a_batch % 32 != 0 ||
                             p->lda < (p->n_tiles - 1u) / p->segment_tiles * p->a_batch + (uint64_t)p->k_tiles * 32u))
        return -3;
    if (k_parts > 1u && (p->epilogue != M40LLM_PACKED_STORE || p->batches != 1u || (k_parts - 1) * part_tiles >= p->k_tiles)) return -3;
    // packed results: whole tiles of columns
    if ((p->epilogue == M40LLM_PACKED_GATED || p->epilogue == M40LLM_PACKED_ROTATE || p->epilogue == M40LLM_PACKED_SILU || p->epilogue == M40LLM_PACKED_SPLIT || p->epilogue == M40LLM_PACKED_TANH ||
         (p->epilogue == M40LLM_PACKED_PROJECT && p->out_act)) &&
        (p->ld_act % 32 != 0 || p->act_col % 4 != 0))
        return -3;
    const bool wide_stores = p->ld_act % 4 == 0 && reinterpret_cast<uintptr_t>(p->out_act) % (p->act_dtype == M40LLM_ACT_F32 ? 16 : 8) == 0;
    switch (p->epilogue) {
        case M40LLM_PACKED_CAP: if (p->batches != 1u || !(p->out_cap >= 0.0f)) return -4; [[fallthrough]];
        case M40LLM_PACKED_STORE: case M40LLM_PACKED_ADD: if (!p->out_f32 || p->cols > p->n_tiles * 16u) return -4; break;
        case M40LLM_PACKED_STORE_ACT: if (!p->out_act || p->cols > p->n_tiles * 16u) return -4; break;
        case M40LLM_PACKED_GATED: if (!p->out_act || !p->gate || p->cols > p->n_tiles * 16u) return -4; break;
        case M40LLM_PACKED_ROTATE:
            if (!p->out_act || !p->angles || p->head_width == 0 || p->head_width % 32 != 0 || p->rot_start % 32 != 0 ||
                p->rot_start >= p->head_width || p->rot_half * 2u != p->head_width - p->rot_start ||
                p->heads * p->head_width != p->n_tiles * 16u || !wide_stores || !m40_aligned16(p->angles) ||
                (p->split_row > 0 && (!p->rot_out || p->ld_rot % 4 != 0 ||
                                      reinterpret_cast<uintptr_t>(p->rot_out) % (p->act_dtype == M40LLM_ACT_F32 ? 16 : 8) != 0)))
                return -4;
            break;
        case M40LLM_PACKED_PROJECT:
            if ((p->plain_tiles > 0 && !p->out_f32) || (p->n_tiles > p->plain_tiles && (!p->out_act || !wide_stores)) ||
                p->plain_tiles % 2 != 0 || p->n_tiles % 2 != 0 || p->plain_tiles > p->n_tiles)
                return -4;
            break;
        case M40LLM_PACKED_SILU: case M40LLM_PACKED_SPLIT: case M40LLM_PACKED_TANH:
            if ((p->plain_tiles > 0 && !p->out_f32) || !p->out_act || !wide_stores || p->plain_tiles > p->n_tiles || p->batches != 1u) return -4;
            break;
        case M40LLM_PACKED_KEYS: case M40LLM_PACKED_VALUES:
            if (!p->out_act || !m40_aligned16(p->out_act) || !p->pages || p->page_k_tiles < p->k_tiles || p->batches != 1u ||
                p->act_dtype != M40LLM_ACT_BF16 || p->rows % M40LLM_PAGE_TOKENS != 0 ||
                (p->epilogue == M40LLM_PACKED_KEYS && p->n_tiles % 2 != 0))
                return -4;
            break;
    }
    PackedArgs g{};
    g.a = p->a;
    g.w = static_cast<const m40_bf16*>(p->w);
    g.lda = (long)p->lda; g.a_batch = (long)p->a_batch * 16; g.w_batch = (long)p->w_batch;
    g.n_tiles = (int)p->n_tiles; g.k_tiles = (int)p->k_tiles; g.rows = (int)p->rows; g.k_stride = (int)p->k_tiles;
    g.pages = p->pages; g.page_k_tiles = (int)p->page_k_tiles;
    g.segment = (int)p->segment_tiles;
    int batches = (int)p->batches;
    if (k_parts > 1u) {
        g.k_total = (int)p->k_tiles; g.k_tiles = (int)part_tiles;
        g.a_batch = (long)part_tiles * kM40Tile; g.w_batch = (long)part_tiles * kM40Tile;
        batches = (int)k_parts;
    }
    (void)hipGetLastError();
    if (p->jobs) {
        g.jobs = p->jobs; g.gather = p->gather;
        g.rows = (int)p->max_jobs;
        const int rows = (int)p->job_rows;
        if (p->act_dtype == M40LLM_ACT_F32) {
            const M40Epilogue<float> e = make_epilogue<float>(*p);
            return p->gather ? launch_rows_any<float, kJobGather>(stream, g, e, 1, rows) : launch_rows_any<float, kJobSlots>(stream, g, e, 1, rows);
        }
        const M40Epilogue<m40_bf16> e = make_epilogue<m40_bf16>(*p);
        if (rows == 128) return launch_tile_any<kSlots>(stream, g, e, 1, ctx->num_cus);
        return p->gather ? launch_rows_any<m40_bf16, kJobGather>(stream, g, e, 1, rows) : launch_rows_any<m40_bf16, kJobSlots>(stream, g, e, 1, rows);
    }
    if (p->act_dtype == M40LLM_ACT_F32) {
        if ((g.rows + 63) / 64 > 65535) return -3;
        return launch_rows_any<float, kAllRows>(stream, g, make_epilogue<float>(*p), batches, g.rows);
    }
    const M40Epilogue<m40_bf16> e = make_epilogue<m40_bf16>(*p);
    if (p->epilogue == M40LLM_PACKED_KEYS) return launch_tile_any<kPageKeys>(stream, g, e, batches, ctx->num_cus);
    if (p->epilogue == M40LLM_PACKED_VALUES) return launch_tile_any<kPageValues>(stream, g, e, batches, ctx->num_cus);
    // few columns leave most CUs without a wide tile
    if (g.rows <= 64 || (g.n_tiles <= 8 && batches == 1 && g.rows <= 65535 * 16 && p->epilogue != M40LLM_PACKED_PROJECT)) return launch_rows_any<m40_bf16, kAllRows>(stream, g, e, batches, g.rows);
    return launch_tile_any<kPlainRows>(stream, g, e, batches, ctx->num_cus);
}

}  // extern "C"
