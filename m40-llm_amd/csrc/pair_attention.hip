// Attention over a paged cache of keys and values (include/m40llm.h has the page order), in kernels for one or two maps a head (M).
// Two maps, differential attention: softmaxes of their own queries and keys over the same values; the second map's result is taken off the
// first's, lambda times, and what is left is normed over the head's value dimensions and gated.  One map: softmax attention, its result
// scaled and, where there is a gate, gated column by column.  One map in the extended form (X): scores capped by a tanh, less a slope times the
// distance of key and query, within a window of the newest tokens, beside a sink in the denominator; all of these are optional.  Scores under a
// small cap need no maximum (kBounded): weights are powers of two of the scores as they are; where the caller also bounds the products of queries and
// keys well inside the cap (kInner), the tanh is a polynomial.
//
// Products are formed transposed, S' = K Q' and O' = V' P': a lane holds the scores of one query (lane % 16) for keys 4 g + r of every
// 16, and pages hold values with their tokens in exactly that order, so the weights a lane computes are its operand of the second
// product, and maximum, sum and rescaling are one value a lane and map.  A kv head's queries are the (row, head of its group) pairs.
//
// pair_rows_kernel   up to 16 queries: every wave takes whole pages straight from memory into operand registers; the waves' sums, and
//                    those of the workgroups that share a sequence's pages (pair_join_kernel), meet at the end
// pair_tile_kernel   64 or 128 queries, a wave 16 or 32 of them: pages go through LDS, one ahead.  With two groups of four waves the even and
//                    the odd pages are walked side by side and the groups' sums meet at the end, which halves the longest walk
// pair_f32_kernel    one workgroup a row and head, plain f32 arithmetic
//
// Maxima are reference points that move only when some score lies 8 (as a power of two) above them.  The sink joins once, when everything is summed.
#include "pair_cache.hpp"

namespace {

constexpr int kPage = M40LLM_PAGE_TOKENS;
constexpr float kLog2e = 1.4426950408889634f;
constexpr float kNothing = -1e30f;         // reference of a row that has seen nothing

struct PairArgs {
    M40llmPairAttention a;
    M40PairPage page;
    uint32_t group;
    float* partial_o;      // [splits][rows * heads][maps][16 v_tiles]
    float* partial_ml;     // [splits][rows * heads][maps][2]: reference, sum
};

// Window of the newest tokens (all: more than there can be), the first page that a query at `pos` sees, and whether every query of a range
// sees the whole page.
__device__ __forceinline__ uint32_t window_of(const M40llmPairAttention& a) { return a.window ? a.window : 0x7fffffffu; }
enum Scores { kPlain = 0, kExtended = 1, kBounded = 2, kInner = 3 };
constexpr float kInnerRange = 0.5f;        // of the tanh's argument
constexpr float kBoundedCap = 60.0f;       // of a score as a power of two: sums of 2^60 and products with values stay far inside f32
template <int X>
__device__ __forceinline__ uint32_t first_page(const M40llmPairAttention& a, uint32_t pos) {
    const uint32_t w = window_of(a);
    return X && pos + 1u > w ? (pos + 1u - w) / kPage : 0u;
}
template <int X>
__device__ __forceinline__ bool whole_page(const M40llmPairAttention& a, uint32_t page, uint32_t first_pos, uint32_t last_pos) {
    return page * kPage + kPage - 1u <= first_pos && (!X || page * kPage + window_of(a) > last_pos);
}
// one over the sum l of weights relative to 2^ref, the sink's included
__device__ __forceinline__ float inverse_sum(const M40llmPairAttention& a, uint32_t head, float ref, float l) {
    if (!a.sink) return 1.0f / l;
    const float sink = static_cast<const float*>(a.sink)[head] * kLog2e, to = fmaxf(ref, sink), f = __builtin_amdgcn_exp2f(ref - to);
    return f / (l * f + __builtin_amdgcn_exp2f(sink - to));
}

// what o (map 1's sums times f1 less map 2's times f2) is multiplied by: sum of squares of o over the head's dimensions in ss
__device__ __forceinline__ float last_factor(const M40llmPairAttention& a, float ss, uint32_t row, uint32_t head) {
    const float z = static_cast<const float*>(a.gate)[(size_t)row * a.ld_gate + head];
    return a.out_scale * m40_sigmoid(z) / sqrtf(ss / (float)a.vdim + a.eps);
}
// one map: what column v of a head's result is multiplied by
__device__ __forceinline__ float column_factor(const M40llmPairAttention& a, uint32_t row, uint32_t head, uint32_t v) {
    return a.gate ? a.out_scale * m40_sigmoid(static_cast<const float*>(a.gate)[(size_t)row * a.ld_gate + head * a.vdim + v]) : a.out_scale;
}

// One page (its tiles at `keys` / `values`, a kilobyte a tile, lane offset included) for B blocks of 16 queries.
template <int M, int DKT, int DVT, int B>
struct PairState {
    m40_bf16x8 q[M][B][DKT];
    m40_float4 o[M][DVT][B];
    float ref[M][B], sum[M][B];
    uint32_t pos[B];

    __device__ __forceinline__ void clear(float reference) {
#pragma unroll
        for (int m = 0; m < M; ++m)
#pragma unroll
            for (int b = 0; b < B; ++b) {
                ref[m][b] = reference;
                sum[m][b] = 0.0f;
#pragma unroll
                for (int j = 0; j < DVT; ++j) o[m][j][b] = m40_float4{0.f, 0.f, 0.f, 0.f};
            }
    }
    // X: products of queries and keys become powers of two that weigh() takes as they are
    __device__ __forceinline__ void extend(const M40llmPairAttention& a, const float (&slope)[B], m40_float4 (&s)[4][B], bool whole, uint32_t key0) const {
        const float window = (float)window_of(a), c = a.cap > 0.0f ? a.scale * 2.0f * kLog2e / a.cap : a.scale * kLog2e, cap = a.cap * kLog2e;
#pragma unroll
        for (int b = 0; b < B; ++b) {
            const float back = (float)((int)key0 - (int)pos[b]);
            if (a.cap > 0.0f) {              // cap tanh(x) = cap - 2 cap / (1 + exp(2 x))
#pragma unroll
                for (int t = 0; t < 4; ++t)
#pragma unroll
                    for (int r = 0; r < 4; ++r) s[t][b][r] = fmaf(-2.0f * cap, __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(s[t][b][r] * c)), cap);
            } else {
#pragma unroll
                for (int t = 0; t < 4; ++t) s[t][b] *= c;
            }
#pragma unroll
            for (int t = 0; t < 4; ++t)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const float d = back + (float)(t * 16 + r);
                    s[t][b][r] = fmaf(slope[b], d, s[t][b][r]);
                    if (!whole) s[t][b][r] = d <= 0.0f && d > -window ? s[t][b][r] : -INFINITY;
                }
        }
    }
    // kBounded, kInner: extend() and weigh() in one, without a reference
    template <int X>
    __device__ __forceinline__ void weigh_bounded(const M40llmPairAttention& a, const float (&slope)[B], m40_float4 (&s)[4][B], bool whole, uint32_t key0, m40_bf16x8 (&pf)[B][2]) {
        const float window = (float)window_of(a), c = a.scale * 2.0f * kLog2e / a.cap, cap = a.cap * kLog2e;
        // kInner: cap tanh(x) as x times a polynomial in x^2, fitted to 1.3e-7 on [-1/2, 1/2], in powers of the product s (x = s scale / cap)
        const float x = a.scale / a.cap, x2 = x * x, p0 = cap * x, k0 = 0.9999976762f * p0, k1 = -0.3332065518f * p0 * x2, k2 = 0.1314514537f * p0 * x2 * x2,
                    k3 = -0.04337247714f * p0 * x2 * x2 * x2;
#pragma unroll
        for (int b = 0; b < B; ++b) {
            const float back = (float)((int)key0 - (int)pos[b]), base = fmaf(slope[b], back, X == kInner ? 0.0f : cap);
            float l = 0.0f;
#pragma unroll
            for (int t = 0; t < 4; ++t)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const float z = s[t][b][r], bias = fmaf(slope[b], (float)(t * 16 + r), base);
                    float e;
                    if (X == kInner) {
                        const float u = z * z;
                        e = __builtin_amdgcn_exp2f(fmaf(z, fmaf(u, fmaf(u, fmaf(u, k3, k2), k1), k0), bias));
                    } else {
                        e = __builtin_amdgcn_exp2f(fmaf(-2.0f * cap, __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(z * c)), bias));
                    }
                    if (!whole) {
                        const float d = back + (float)(t * 16 + r);
                        e = d <= 0.0f && d > -window ? e : 0.0f;
                    }
                    l += e;
                    pf[b][t >> 1][(t & 1) * 4 + r] = static_cast<m40_bf16>(e);
                }
            sum[0][b] += l;
        }
    }
    // the scores of a map become weights: operands of the value product
    __device__ __forceinline__ void weigh(int m, m40_float4 (&s)[4][B], float c, bool whole, uint32_t key0, m40_bf16x8 (&pf)[B][2]) {
        if (!whole) {
#pragma unroll
            for (int b = 0; b < B; ++b)
#pragma unroll
                for (int t = 0; t < 4; ++t)
#pragma unroll
                    for (int r = 0; r < 4; ++r) s[t][b][r] = key0 + t * 16 + r <= pos[b] ? s[t][b][r] : -INFINITY;
        }
#pragma unroll
        for (int b = 0; b < B; ++b) {
            float top = fmaxf(fmaxf(s[0][b][0], s[0][b][1]), fmaxf(s[0][b][2], s[0][b][3]));
#pragma unroll
            for (int t = 1; t < 4; ++t) top = fmaxf(top, fmaxf(fmaxf(s[t][b][0], s[t][b][1]), fmaxf(s[t][b][2], s[t][b][3])));
            top *= c;
            if (__any(top > ref[m][b] + 8.0f)) {
                top = m40_max_xor16(top);
                top = m40_max_xor32(top);
                const float to = fmaxf(ref[m][b], top), f = __builtin_amdgcn_exp2f(ref[m][b] - to);
                ref[m][b] = to;
                sum[m][b] *= f;
#pragma unroll
                for (int j = 0; j < DVT; ++j) o[m][j][b] *= f;
            }
            const float less = -ref[m][b];
            float l = 0.0f;
#pragma unroll
            for (int t = 0; t < 4; ++t)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const float e = __builtin_amdgcn_exp2f(fmaf(s[t][b][r], c, less));
                    l += e;
                    pf[b][t >> 1][(t & 1) * 4 + r] = static_cast<m40_bf16>(e);
                }
            sum[m][b] += l;
        }
    }
    // joins sums of other keys (reference, sum and weighted values given as functions of their place)
    template <class G>
    __device__ __forceinline__ void join(G get) {
#pragma unroll
        for (int m = 0; m < M; ++m)
#pragma unroll
            for (int b = 0; b < B; ++b) {
                const int at = (m * B + b) * (2 + 4 * DVT);
                const float other = get(at), to = fmaxf(ref[m][b], other);
                const float f0 = __builtin_amdgcn_exp2f(ref[m][b] - to), f1 = __builtin_amdgcn_exp2f(other - to);
                ref[m][b] = to;
                sum[m][b] = sum[m][b] * f0 + get(at + 1) * f1;
#pragma unroll
                for (int j = 0; j < DVT; ++j)
#pragma unroll
                    for (int r = 0; r < 4; ++r) o[m][j][b][r] = o[m][j][b][r] * f0 + get(at + 2 + j * 4 + r) * f1;
            }
    }
    static constexpr int kFloats = M * B * (2 + 4 * DVT);       // of a lane
    template <class P>
    __device__ __forceinline__ void put(P set) const {
#pragma unroll
        for (int m = 0; m < M; ++m)
#pragma unroll
            for (int b = 0; b < B; ++b) {
                const int at = (m * B + b) * (2 + 4 * DVT);
                set(at, ref[m][b]);
                set(at + 1, sum[m][b]);
#pragma unroll
                for (int j = 0; j < DVT; ++j)
#pragma unroll
                    for (int r = 0; r < 4; ++r) set(at + 2 + j * 4 + r, o[m][j][b][r]);
            }
    }
    // the result of query block b to its row
    __device__ __forceinline__ void finish(const PairArgs& p, int b, uint32_t row, uint32_t head, bool live, int g) const {
        const int vt = (int)p.page.v_tiles, vdim = (int)p.a.vdim;
        const float l = m40_add_xor32(m40_add_xor16(sum[0][b])), f1 = M == 1 ? inverse_sum(p.a, head, ref[0][b], l) : 1.0f / l;
        if constexpr (M == 1) {
            if (!live) return;
            const bool vec = p.a.gate && vdim % 4 == 0 && p.a.ld_gate % 4 == 0 && m40_aligned16(p.a.gate);
            const float* gate = static_cast<const float*>(p.a.gate) + (p.a.gate ? (size_t)row * p.a.ld_gate + head * vdim : 0);
#pragma unroll
            for (int j = 0; j < DVT; ++j) {
                const int v = j * 16 + 4 * g;
                if (j >= vt || v >= vdim) continue;
                m40_float4 y = o[0][j][b] * f1;
                if (vec) {
                    const m40_float4 z = *reinterpret_cast<const m40_float4*>(gate + v);
#pragma unroll
                    for (int r = 0; r < 4; ++r) y[r] *= p.a.out_scale * m40_sigmoid(z[r]);
                } else {
#pragma unroll
                    for (int r = 0; r < 4; ++r) y[r] *= column_factor(p.a, row, head, (uint32_t)(v + r < vdim ? v + r : vdim - 1));
                }
                m40_store_packed<m40_bf16>(static_cast<m40_bf16*>(p.a.out), (int)row, (int)head * vdim + v, (long)p.a.ld_out, y, vdim - v, vdim % 4 == 0);
            }
        } else {
        const float f2 = p.a.lambda / m40_add_xor32(m40_add_xor16(sum[M - 1][b]));
        float ss = 0.0f;
        m40_float4 d[DVT];
#pragma unroll
        for (int j = 0; j < DVT; ++j) {
            d[j] = o[0][j][b] * f1 - o[M - 1][j][b] * f2;       // dimensions past vdim are zero in every page
            if (j < vt) ss += d[j][0] * d[j][0] + d[j][1] * d[j][1] + d[j][2] * d[j][2] + d[j][3] * d[j][3];
        }
        ss = m40_add_xor32(m40_add_xor16(ss));
        if (!live) return;
        const float f = last_factor(p.a, ss, row, head);
#pragma unroll
        for (int j = 0; j < DVT; ++j) {
            const int v = j * 16 + 4 * g;
            if (j < vt && v < vdim)
                m40_store_packed<m40_bf16>(static_cast<m40_bf16*>(p.a.out), (int)row, (int)head * vdim + v, (long)p.a.ld_out, d[j] * f, vdim - v, vdim % 4 == 0);
        }
        }
    }
};

// what a power of two loses per token of distance
__device__ __forceinline__ float slope_of(const M40llmPairAttention& a, uint32_t head) { return a.slopes ? static_cast<const float*>(a.slopes)[head] * kLog2e : 0.0f; }

template <int M, int DKT, int DVT, int X>
__global__ __launch_bounds__(256, 1) void pair_rows_kernel(PairArgs p) {
    extern __shared__ __align__(16) float join_lds[];      // three waves' sums
    const M40llmPairAttention& a = p.a;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), g = lane >> 4, li = lane & 15;
    const int kt = (int)p.page.k_tiles, vt = (int)p.page.v_tiles;
    const uint32_t q0 = a.tiles[2 * blockIdx.x], count = a.tiles[2 * blockIdx.x + 1], kv = blockIdx.y;
    const bool live = (uint32_t)li < count;
    const uint32_t query = q0 + (live ? (uint32_t)li : count - 1u), row = query / p.group, head = kv * p.group + query % p.group;
    const uint32_t last_row = (q0 + count - 1u) / p.group;
    const uint32_t first_pos = a.row_pos[q0 / p.group], last_pos = a.row_pos[last_row];
    const uint32_t pages = last_pos / kPage + 1u, skipped = first_page<X>(a, first_pos), per = (pages - skipped + a.splits - 1u) / a.splits;
    const uint32_t page0 = skipped + blockIdx.z * per, page1 = page0 + per < pages ? page0 + per : pages;
    const uint32_t* table = a.page_table + (size_t)a.row_slot[last_row] * a.max_pages;
    PairState<M, DKT, DVT, 1> s;
    s.clear(X >= kBounded ? 0.0f : kNothing);
    s.pos[0] = a.row_pos[row];
    const float slope[1] = {X ? slope_of(a, head) : 0.0f};
    const m40_bf16* q = static_cast<const m40_bf16*>(a.queries) + ((size_t)row * a.heads + head) * ((uint32_t)M * kt * 32u) + g * 8;
#pragma unroll
    for (int m = 0; m < M; ++m)
#pragma unroll
        for (int k = 0; k < DKT; ++k) {
            s.q[m][0][k] = *reinterpret_cast<const m40_bf16x8*>(q + (m * kt + (k < kt ? k : kt - 1)) * 32);
            if (k >= kt) s.q[m][0][k] = m40_bf16x8{};      // key tiles past the head's are read again and count nothing
        }
    const float c = a.scale * kLog2e;
    const m40_bf16* cache = static_cast<const m40_bf16*>(a.cache) + kv * p.page.head_elements() + lane * 8;
    for (uint32_t n = page0 + wave; n < page1; n += 4u) {
        const m40_bf16* keys = cache + table[n] * p.page.elements();
        const m40_bf16* values = keys + p.page.key_elements();
        const bool whole = whole_page<X>(a, n, first_pos, last_pos);
        m40_bf16x8 pf[M][1][2], vf[DVT][2];
#pragma unroll
        for (int m = 0; m < M; ++m) {
            m40_float4 sc[4][1];
#pragma unroll
            for (int t = 0; t < 4; ++t) {
                sc[t][0] = m40_float4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int k = 0; k < DKT; ++k) {
                    const m40_bf16x8 kf = *reinterpret_cast<const m40_bf16x8*>(keys + ((m * 4 + t) * kt + (k < kt ? k : kt - 1)) * kM40Tile);
                    sc[t][0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, s.q[m][0][k], sc[t][0], 0, 0, 0);
                }
            }
            if (m == 0) {
#pragma unroll
                for (int j = 0; j < DVT; ++j)
#pragma unroll
                    for (int h = 0; h < 2; ++h) vf[j][h] = *reinterpret_cast<const m40_bf16x8*>(values + ((j < vt ? j : vt - 1) * 2 + h) * kM40Tile);
            }
            if constexpr (X >= kBounded) {
                s.template weigh_bounded<X>(a, slope, sc, whole, n * kPage + 4 * g, pf[m]);
            } else {
                if constexpr (X == kExtended) s.extend(a, slope, sc, whole, n * kPage + 4 * g);
                s.weigh(m, sc, X ? 1.0f : c, X || whole, n * kPage + 4 * g, pf[m]);
            }
        }
#pragma unroll
        for (int j = 0; j < DVT; ++j)
#pragma unroll
            for (int m = 0; m < M; ++m)
#pragma unroll
                for (int h = 0; h < 2; ++h) s.o[m][j][0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[j][h], pf[m][0][h], s.o[m][j][0], 0, 0, 0);
    }
    constexpr int kFloats = PairState<M, DKT, DVT, 1>::kFloats;
    if (wave > 0) {
        float* mine = join_lds + (size_t)(wave - 1) * kFloats * 64 + lane;
        s.put([&](int i, float v) { mine[i * 64] = v; });
    }
    __syncthreads();
    if (wave > 0) return;
#pragma unroll
    for (int w = 0; w < 3; ++w) {
        const float* other = join_lds + (size_t)w * kFloats * 64 + lane;
        s.join([&](int i) { return other[i * 64]; });
    }
    if (a.splits == 1u) {
        s.finish(p, 0, row, head, live, g);
        return;
    }
    float l[M];
#pragma unroll
    for (int m = 0; m < M; ++m) l[m] = m40_add_xor32(m40_add_xor16(s.sum[m][0]));
    if (!live) return;
    const size_t at = (size_t)blockIdx.z * a.n_rows * a.heads + (size_t)(row - a.first_row) * a.heads + head;
#pragma unroll
    for (int m = 0; m < M; ++m) {
        if (g == 0) {
            p.partial_ml[(at * M + m) * 2] = s.ref[m][0];
            p.partial_ml[(at * M + m) * 2 + 1] = l[m];
        }
#pragma unroll
        for (int j = 0; j < DVT; ++j)
            if (j < vt) *reinterpret_cast<m40_float4*>(p.partial_o + ((at * M + m) * vt + j) * 16 + 4 * g) = s.o[m][j][0];
    }
}

// A workgroup a row and head: the splits' weights first, then eight groups of 32 lanes take every eighth split.
constexpr int kJoinSplits = 256;
template <class T, int M>
__global__ __launch_bounds__(256) void pair_join_kernel(PairArgs p) {
    __shared__ float weight[M][kJoinSplits];
    __shared__ m40_float4 sums[8][32];
    __shared__ float part[4];
    __shared__ float o_lds[M][M40LLM_PAIR_MOST_DIM];
    const M40llmPairAttention& a = p.a;
    const uint32_t i = blockIdx.x, row = a.first_row + i / a.heads, head = i % a.heads, tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6;
    const uint32_t width = p.page.v_tiles * 16u, group = tid >> 5;
    const size_t stride = (size_t)a.n_rows * a.heads;
    for (uint32_t m = 0; m < (uint32_t)M; ++m) {
        const float* ml = p.partial_ml + ((size_t)i * M + m) * 2u;
        const float ref = tid < a.splits ? ml[tid * stride * 2u * M] : kNothing, l = tid < a.splits ? ml[tid * stride * 2u * M + 1u] : 0.0f;
        const float top = m40_max64(ref);
        if (lane == 0) part[wave] = top;
        __syncthreads();
        const bool sunk = M == 1 && a.sink;
        const float sink = sunk ? static_cast<const float*>(a.sink)[head] * kLog2e : kNothing;
        const float to = fmaxf(fmaxf(fmaxf(part[0], part[1]), fmaxf(part[2], part[3])), sink);
        const float e = __builtin_amdgcn_exp2f(ref - to), den = m40_sum64(l * e);
        __syncthreads();
        if (tid < a.splits) weight[m][tid] = e;
        if (lane == 0) part[wave] = den;
        __syncthreads();
        const float inv = (m ? -a.lambda : 1.0f) / (part[0] + part[1] + part[2] + part[3] + (sunk ? __builtin_amdgcn_exp2f(sink - to) : 0.0f));
        for (uint32_t d0 = 0; d0 < width; d0 += 128u) {
            const uint32_t d = d0 + (tid & 31u) * 4u;
            m40_float4 acc = {0.f, 0.f, 0.f, 0.f};
            if (d < width) {
                const float* o = p.partial_o + ((size_t)i * M + m) * width + d;
#pragma unroll 4
                for (uint32_t s = group; s < a.splits; s += 8u) acc += *reinterpret_cast<const m40_float4*>(o + s * stride * M * width) * weight[m][s];
            }
            sums[group][tid & 31u] = acc;
            __syncthreads();
            if (group == 0 && d < width) {
#pragma unroll
                for (int k = 1; k < 8; ++k) acc += sums[k][tid & 31u];
#pragma unroll
                for (int k = 0; k < 4; ++k) o_lds[m][d + k] = acc[k] * inv;
            }
            __syncthreads();
        }
    }
    if constexpr (M == 1) {
        if (tid < a.vdim)
            static_cast<T*>(a.out)[m40_packed_at(row, head * a.vdim + tid, a.ld_out >> 5)] = M40Act<T>::from(o_lds[0][tid] * column_factor(a, row, head, tid));
        return;
    }
    const float o = tid < a.vdim ? o_lds[0][tid] + o_lds[M - 1][tid] : 0.0f;
    const float ss = m40_sum64(o * o);
    if (lane == 0) part[wave] = ss;
    __syncthreads();
    const float f = last_factor(a, part[0] + part[1] + part[2] + part[3], row, head);
    if (tid < a.vdim) static_cast<T*>(a.out)[m40_packed_at(row, head * a.vdim + tid, a.ld_out >> 5)] = M40Act<T>::from(o * f);
}

template <int M, int DKT, int DVT, int QB, int GROUPS, int PER_CU, int X>
__global__ __launch_bounds__(GROUPS * 256, PER_CU) void pair_tile_kernel(PairArgs p) {
    typedef __attribute__((address_space(3))) void* lds_dst_t;
    typedef const __attribute__((address_space(1))) void* global_src_t;
    extern __shared__ __align__(16) uint8_t lds[];
    const M40llmPairAttention& a = p.a;
    const int lane = threadIdx.x & 63, w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), g = lane >> 4, li = lane & 15;
    const int wave = w & 3, group = w >> 2;
    const int kt = (int)p.page.k_tiles, vt = (int)p.page.v_tiles, page_tiles = 4 * M * kt + 2 * vt;
    const uint32_t kv = blockIdx.x, q0 = a.tiles[2 * blockIdx.y], count = a.tiles[2 * blockIdx.y + 1];
    const uint32_t last_row = (q0 + count - 1u) / p.group;
    const uint32_t last = a.row_pos[last_row] / kPage, skipped = first_page<X>(a, a.row_pos[q0 / p.group]), pages = last + 1u - skipped;
    const uint32_t* table = a.page_table + (size_t)a.row_slot[last_row] * a.max_pages;
    const m40_bf16* cache = static_cast<const m40_bf16*>(a.cache) + kv * p.page.head_elements() + lane * 8;
    // a kv head's part of a page is contiguous: keys, then values
    auto issue = [&](int buf, uint32_t number) __attribute__((always_inline)) {
        const m40_bf16* src = cache + number * p.page.elements();
        for (int i = wave; i < page_tiles; i += 4)
            __builtin_amdgcn_global_load_lds((global_src_t)(src + (size_t)i * kM40Tile), (lds_dst_t)(lds + ((group * 2 + buf) * page_tiles + i) * 1024), 16, 0, 0);
    };
    const uint32_t steps = (pages + GROUPS - 1u) / GROUPS;
    auto page_of = [&](uint32_t step) { const uint32_t n = skipped + step * GROUPS + group; return n < last ? n : last; };    // past the end: the last again
    issue(0, table[page_of(0)]);
    uint32_t next = table[page_of(1)];
    PairState<M, DKT, DVT, QB> s;
    s.clear(X >= kBounded ? 0.0f : kNothing);
    uint32_t row[QB], head[QB];
    bool live[QB];
#pragma unroll
    for (int b = 0; b < QB; ++b) {
        const uint32_t i = (uint32_t)(wave * 16 * QB + b * 16 + li);
        live[b] = i < count;
        const uint32_t query = q0 + (live[b] ? i : count - 1u);
        row[b] = query / p.group;
        head[b] = kv * p.group + query % p.group;
        s.pos[b] = a.row_pos[row[b]];
        const m40_bf16* q = static_cast<const m40_bf16*>(a.queries) + ((size_t)row[b] * a.heads + head[b]) * ((uint32_t)M * kt * 32u) + g * 8;
#pragma unroll
        for (int m = 0; m < M; ++m)
#pragma unroll
            for (int k = 0; k < DKT; ++k) {
                s.q[m][b][k] = *reinterpret_cast<const m40_bf16x8*>(q + (m * kt + (k < kt ? k : kt - 1)) * 32);
                if (k >= kt) s.q[m][b][k] = m40_bf16x8{};
            }
    }
    // the wave's first and last positions: pages past the last are not worked on, pages up to the first need no compares
    const uint32_t i_first = (uint32_t)wave * 16u * QB, i_last = i_first + 16u * QB - 1u;
    const bool wave_live = i_first < count;
    const uint32_t pos_first = a.row_pos[(q0 + (wave_live ? i_first : count - 1u)) / p.group], pos_last = a.row_pos[(q0 + (i_last < count ? i_last : count - 1u)) / p.group];
    const float c = a.scale * kLog2e;
    float slope[QB];
#pragma unroll
    for (int b = 0; b < QB; ++b) slope[b] = X ? slope_of(a, head[b]) : 0.0f;
    int buf = 0;
    for (uint32_t step = 0; step < steps; ++step, buf ^= 1) {
        m40_wait_and_meet<0>();                  // the pages have landed, and nobody reads the other buffers any more
        if (step + 1u < steps) {
            issue(buf ^ 1, next);
            next = table[page_of(step + 2u)];
        }
        const uint32_t n = skipped + step * GROUPS + group;
        if (!wave_live || n > last || n * kPage > pos_last || (X && n < first_page<X>(a, pos_first))) continue;
        const uint8_t* keys = lds + (group * 2 + buf) * page_tiles * 1024 + lane * 16;
        const uint8_t* values = keys + 4 * M * kt * 1024;
        const bool whole = whole_page<X>(a, n, pos_first, pos_last);
        m40_bf16x8 pf[M][QB][2];
#pragma unroll
        for (int m = 0; m < M; ++m) {
            m40_float4 sc[4][QB];
#pragma unroll
            for (int t = 0; t < 4; ++t)
#pragma unroll
                for (int b = 0; b < QB; ++b) sc[t][b] = m40_float4{0.f, 0.f, 0.f, 0.f};
            __builtin_amdgcn_s_setprio(1);
#pragma unroll
            for (int k = 0; k < DKT; ++k)
                if (k < kt) {
#pragma unroll
                    for (int t = 0; t < 4; ++t) {
                        const m40_bf16x8 kf = *reinterpret_cast<const m40_bf16x8*>(keys + ((m * 4 + t) * kt + k) * 1024);
#pragma unroll
                        for (int b = 0; b < QB; ++b) sc[t][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, s.q[m][b][k], sc[t][b], 0, 0, 0);
                    }
                }
            __builtin_amdgcn_s_setprio(0);
            if constexpr (X >= kBounded) {
                s.template weigh_bounded<X>(a, slope, sc, whole, n * kPage + 4 * g, pf[m]);
            } else {
                if constexpr (X == kExtended) s.extend(a, slope, sc, whole, n * kPage + 4 * g);
                s.weigh(m, sc, X ? 1.0f : c, X || whole, n * kPage + 4 * g, pf[m]);
            }
        }
        __builtin_amdgcn_s_setprio(1);
#pragma unroll
        for (int j = 0; j < DVT; ++j)
            if (j < vt) {
#pragma unroll
                for (int h = 0; h < 2; ++h) {
                    const m40_bf16x8 vf = *reinterpret_cast<const m40_bf16x8*>(values + (j * 2 + h) * 1024);
#pragma unroll
                    for (int m = 0; m < M; ++m)
#pragma unroll
                        for (int b = 0; b < QB; ++b) s.o[m][j][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[m][b][h], s.o[m][j][b], 0, 0, 0);
                }
            }
        __builtin_amdgcn_s_setprio(0);
    }
    if constexpr (GROUPS == 2) {
        m40_wait_and_meet<0>();                  // every buffer is free
        float* mine = reinterpret_cast<float*>(lds) + (size_t)wave * PairState<M, DKT, DVT, QB>::kFloats * 64 + lane;
        if (group == 1) s.put([&](int i, float v) { mine[i * 64] = v; });
        m40_wait_and_meet<63>();
        if (group == 1) return;
        s.join([&](int i) { return mine[i * 64]; });
    } else {
        __builtin_amdgcn_s_waitcnt(m40_vm_lgkm_wait(0));
    }
    if (!wave_live) return;
#pragma unroll
    for (int b = 0; b < QB; ++b) s.finish(p, b, row[b], head[b], live[b], g);
}

template <int M>
__global__ __launch_bounds__(256) void pair_f32_kernel(PairArgs p) {
    __shared__ float q[M][M40LLM_PAIR_MOST_DIM], o[M][M40LLM_PAIR_MOST_DIM], s[M][kPage];
    __shared__ float stat[M][3];             // maximum, sum, factor on what came before
    __shared__ float part[4];
    const M40llmPairAttention& a = p.a;
    const uint32_t tid = threadIdx.x, row = a.first_row + blockIdx.x / a.heads, head = blockIdx.x % a.heads, kv = head / p.group;
    const uint32_t width = p.page.k_tiles * 32u;
    for (uint32_t i = tid; i < M * width; i += 256u) q[i / width][i % width] = static_cast<const float*>(a.queries)[((size_t)row * a.heads + head) * M * width + i];
    for (uint32_t i = tid; i < M * a.vdim; i += 256u) o[i / a.vdim][i % a.vdim] = 0.0f;
    if (tid < (uint32_t)M) { stat[tid][0] = -INFINITY; stat[tid][1] = 0.0f; }
    const uint32_t pos = a.row_pos[row], pages = pos / kPage + 1u;
    const uint32_t* table = a.page_table + (size_t)a.row_slot[row] * a.max_pages;
    const float slope = M == 1 && a.slopes ? static_cast<const float*>(a.slopes)[head] : 0.0f;
    __syncthreads();
    for (uint32_t n = first_page<M == 1 ? kExtended : kPlain>(a, pos); n < pages; ++n) {
        const float* page = static_cast<const float*>(a.cache) + table[n] * p.page.elements() + kv * p.page.head_elements();
        // two lanes a token and map of two, four a token of one
        constexpr uint32_t kLanes = 4u / M;
        const uint32_t map = tid / (kPage * kLanes), t = tid / kLanes % kPage;
        float x = 0.0f;
        for (uint32_t d = tid % kLanes; d < a.dim; d += kLanes) x = fmaf(q[map][d], page[p.page.key_at(map, t, d)], x);
        x += m40_dpp_f<M40_DPP_XOR1>(x);
        if (kLanes == 4u) x += m40_dpp_f<M40_DPP_XOR2>(x);
        x *= a.scale;
        if (M == 1) {
            if (a.cap > 0.0f) x = a.cap * tanhf(x / a.cap);
            x -= slope * ((float)pos - (float)(n * kPage + t));
        }
        const uint32_t key = n * kPage + t;
        if (tid % kLanes == 0u) s[map][t] = key <= pos && (M != 1 || pos - key < window_of(a)) ? x : -INFINITY;
        __syncthreads();
        if (tid < 64u * M) {                 // a wave a map; a page of the range holds a seen token
            const uint32_t m = tid >> 6, l = tid & 63u;
            const float v = s[m][l], before = stat[m][0], top = fmaxf(before, m40_max64(v));
            const float e = expf(v - top), f = expf(before - top), sum = m40_sum64(e);
            s[m][l] = e;
            if (l == 0u) { stat[m][0] = top; stat[m][1] = stat[m][1] * f + sum; stat[m][2] = f; }
        }
        __syncthreads();
        for (uint32_t i = tid; i < M * a.vdim; i += 256u) {
            const uint32_t m = i / a.vdim, d = i % a.vdim;
            float acc = o[m][d] * stat[m][2];
            for (uint32_t k = 0; k < (uint32_t)kPage; ++k) acc = fmaf(s[m][k], page[p.page.value_at(k, d)], acc);
            o[m][d] = acc;
        }
        __syncthreads();
    }
    if constexpr (M == 1) {
        float below = stat[0][1], f = 1.0f;
        if (a.sink) {
            const float sink = static_cast<const float*>(a.sink)[head], to = fmaxf(stat[0][0], sink);
            f = expf(stat[0][0] - to);
            below = below * f + expf(sink - to);
        }
        if (tid < a.vdim)
            static_cast<float*>(a.out)[m40_packed_at(row, head * a.vdim + tid, a.ld_out >> 5)] = o[0][tid] * f / below * column_factor(a, row, head, tid);
        return;
    }
    const float y = tid < a.vdim ? o[0][tid] / stat[0][1] - a.lambda * (o[M - 1][tid] / stat[M - 1][1]) : 0.0f;
    const float ss = m40_sum64(y * y);
    if ((tid & 63u) == 0u) part[tid >> 6] = ss;
    __syncthreads();
    const float f = last_factor(a, part[0] + part[1] + part[2] + part[3], row, head);
    if (tid < a.vdim) static_cast<float*>(a.out)[m40_packed_at(row, head * a.vdim + tid, a.ld_out >> 5)] = y * f;
}

constexpr int kLdsMax = 160 * 1024;

template <int M, int DKT, int DVT, int X>
int launch_rows(hipStream_t stream, const PairArgs& p) {
    constexpr int lds = 3 * 64 * 4 * PairState<M, DKT, DVT, 1>::kFloats;
    static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(pair_rows_kernel<M, DKT, DVT, X>), hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    if (attr != hipSuccess) return -2;
    pair_rows_kernel<M, DKT, DVT, X><<<dim3(p.a.n_tiles, p.a.kv_heads, p.a.splits), 256, lds, stream>>>(p);
    return hipGetLastError() == hipSuccess ? 0 : -2;
}
int page_lds(const PairArgs& p, int groups) { return groups * 2 * (int)(4u * p.page.maps * p.page.k_tiles + 2u * p.page.v_tiles) * 1024; }
template <int M, int DKT, int DVT, int QB, int GROUPS, int PER_CU, int X>
int launch_tile(hipStream_t stream, const PairArgs& p) {
    static const hipError_t attr =
        hipFuncSetAttribute(reinterpret_cast<const void*>(pair_tile_kernel<M, DKT, DVT, QB, GROUPS, PER_CU, X>), hipFuncAttributeMaxDynamicSharedMemorySize, kLdsMax);
    if (attr != hipSuccess) return -2;
    constexpr int join = GROUPS == 2 ? 4 * 64 * 4 * PairState<M, DKT, DVT, QB>::kFloats : 0;
    static_assert(join <= kLdsMax, "the joining of two groups does not fit");
    const int pages = page_lds(p, GROUPS);
    pair_tile_kernel<M, DKT, DVT, QB, GROUPS, PER_CU, X><<<dim3(p.a.kv_heads, p.a.n_tiles), GROUPS * 256, pages > join ? pages : join, stream>>>(p);
    return hipGetLastError() == hipSuccess ? 0 : -2;
}
// PER_CU: workgroups of one group a CU that fit
template <int M, int DKT, int DVT, int PER_CU, int X>
int launch_tile_any(hipStream_t stream, const PairArgs& p, int num_cus) {
    // With enough workgroups the short ones fill in behind the long ones.  Where all walks are alike there is nothing to halve, and two workgroups
    // a CU, whose barriers are their own, overlap products and weights better than two groups of one.
    const uint64_t workgroups = (uint64_t)p.a.kv_heads * p.a.n_tiles;
    if (page_lds(p, 2) <= kLdsMax && workgroups <= 3ull * (uint32_t)num_cus && !(p.a.even && workgroups >= 2ull * (uint32_t)num_cus))
        return p.a.tile_queries == 64u ? launch_tile<M, DKT, DVT, 1, 2, PER_CU, X>(stream, p) : launch_tile<M, DKT, DVT, 2, 2, PER_CU, X>(stream, p);
    return p.a.tile_queries == 64u ? launch_tile<M, DKT, DVT, 1, 1, PER_CU, X>(stream, p) : launch_tile<M, DKT, DVT, 2, 1, PER_CU, X>(stream, p);
}

bool tile_served(uint32_t maps, uint32_t k_tiles, uint32_t v_tiles) { return 2u * (4u * maps * k_tiles + 2u * v_tiles) * 1024u <= (uint32_t)kLdsMax; }

// PER_CU of heads of 128 dimensions
template <int M, int PER_CU, int X>
int launch_form(hipStream_t stream, const PairArgs& p, uint32_t form, int num_cus) {
    const uint32_t kt = p.page.k_tiles, vt = p.page.v_tiles;
    if (form == 1u) {
        if (kt <= 2u && vt <= 4u) return launch_tile_any<M, 2, 4, 2, X>(stream, p, num_cus);
        if (kt <= 2u && vt <= 8u) return launch_tile_any<M, 2, 8, 2, X>(stream, p, num_cus);
        if (kt <= 4u && vt <= 8u) return launch_tile_any<M, 4, 8, PER_CU, X>(stream, p, num_cus);
        return launch_tile<M, 8, 16, 1, 1, 1, X>(stream, p);
    }
    if constexpr (X >= kBounded) {               // rows: the extended form hides more of the pages' latency
        return -3;
    } else {
        int rc;
        if (kt <= 2u && vt <= 4u) rc = launch_rows<M, 2, 4, X>(stream, p);
        else if (kt <= 2u && vt <= 8u) rc = launch_rows<M, 2, 8, X>(stream, p);
        else if (kt <= 4u && vt <= 8u) rc = launch_rows<M, 4, 8, X>(stream, p);
        else rc = launch_rows<M, 8, 16, X>(stream, p);
        if (rc != 0 || p.a.splits == 1u) return rc;
        pair_join_kernel<m40_bf16, M><<<p.a.n_rows * p.a.heads, 256, 0, stream>>>(p);
        return hipGetLastError() == hipSuccess ? 0 : -2;
    }
}
int launch(hipStream_t stream, const PairArgs& p, uint32_t form, int num_cus) {
    if (p.a.maps == 2u) return launch_form<2, 1, kPlain>(stream, p, form, num_cus);
    if (form == 1u && p.a.cap > 0.0f && p.a.cap * kLog2e <= kBoundedCap) {
        if (p.a.most > 0.0f && p.a.most * p.a.scale <= kInnerRange * p.a.cap) return launch_form<1, 2, kInner>(stream, p, form, num_cus);
        return launch_form<1, 2, kBounded>(stream, p, form, num_cus);
    }
    if (p.a.window || p.a.cap > 0.0f || p.a.slopes) return launch_form<1, 2, kExtended>(stream, p, form, num_cus);
    return launch_form<1, 2, kPlain>(stream, p, form, num_cus);
}

}  // namespace

extern "C" {

uint64_t m40llm_ext_pair_attention_partial_floats(uint32_t maps, uint32_t rows, uint32_t heads, uint32_t vdim, uint32_t splits) {
    return splits <= 1u ? 0u : (uint64_t)splits * rows * heads * maps * ((vdim + 15u) / 16u * 16u + 2u);
}

uint32_t m40llm_ext_pair_attention_tile_queries(uint32_t act_dtype, uint32_t maps, uint32_t dim, uint32_t vdim) {
    if (maps == 0 || maps > 2u || dim == 0 || vdim == 0 || dim > M40LLM_PAIR_MOST_DIM || vdim > M40LLM_PAIR_MOST_DIM) return 0;
    if (act_dtype == M40LLM_ACT_F32) return 128u;
    const uint32_t kt = (dim + 31u) / 32u, vt = (vdim + 15u) / 16u;
    return !tile_served(maps, kt, vt) ? 16u : vt <= 8u && kt <= 4u ? 128u : 64u;
}

int m40llm_ext_pair_attention_async(M40llmCudaContext* ctx, const M40llmPairAttention* a, uint32_t stream_kind) {
    if (!ctx || !a || !a->queries || !a->cache || (!a->gate && a->maps != 1u) || !a->row_slot || !a->row_pos || !a->page_table || !a->out) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    const uint32_t most = m40llm_ext_pair_attention_tile_queries(a->act_dtype, a->maps, a->dim, a->vdim);
    if (a->act_dtype > 1u || a->form > 1u || a->heads == 0 || a->kv_heads == 0 || a->heads % a->kv_heads != 0 || most == 0 || !(a->scale > 0.0f) || a->ld_out % 32u != 0 ||
        a->ld_out < a->heads * a->vdim || a->n_rows == 0 || !m40_aligned16(a->queries) || !m40_aligned16(a->cache) || a->window > 0x7fffffffu || !(a->cap >= 0.0f) ||
        (a->maps != 1u && (a->window || a->cap > 0.0f || a->slopes || a->sink)))
        return -3;
    PairArgs p{*a, M40PairPage(a->maps, a->kv_heads, a->dim, a->vdim), a->heads / a->kv_heads, nullptr, nullptr};
    (void)hipGetLastError();
    if (a->act_dtype == M40LLM_ACT_F32) {
        if (a->maps == 1u) pair_f32_kernel<1><<<a->n_rows * a->heads, 256, 0, stream>>>(p);
        else pair_f32_kernel<2><<<a->n_rows * a->heads, 256, 0, stream>>>(p);
        return hipGetLastError() == hipSuccess ? 0 : -2;
    }
    if (!a->tiles || a->n_tiles == 0) return -1;
    const uint32_t kt = p.page.k_tiles, vt = p.page.v_tiles;
    if (a->form == 1u) {
        if ((a->tile_queries != 64u && a->tile_queries != 128u) || a->tile_queries > most || a->n_tiles > 65535u || !tile_served(a->maps, kt, vt)) return -3;
        return launch(stream, p, 1u, ctx->num_cus);
    }
    if (a->splits == 0 || a->splits > (uint32_t)kJoinSplits || a->kv_heads > 65535u) return -3;
    if (a->splits > 1u) {
        if (!a->partial || !m40_aligned16(a->partial) ||
            a->partial_floats < m40llm_ext_pair_attention_partial_floats(a->maps, a->n_rows, a->heads, a->vdim, a->splits))
            return -4;
        p.partial_o = static_cast<float*>(a->partial);
        p.partial_ml = p.partial_o + (size_t)a->splits * a->n_rows * a->heads * a->maps * vt * 16u;
    }
    return launch(stream, p, 0u, ctx->num_cus);
}

}  // extern "C"
