// Attention in latent space over a paged cache: every head of a token reads the same cache entries (normed latent, then the
// rotated key part), so the heads of a token -- and of neighbouring tokens of a portion -- are the rows of one matrix tile.
//
// bf16: a workgroup of four waves takes a tile of up to 64 query rows (token, head) and walks its share of the pages.  Per
// page of 64 tokens: the page goes to LDS as it lies in memory; wave w scores the 16 tokens of group w against all rows
// (16x16x32 matrix instruction); the four waves agree on the row maxima; the weights go through LDS; wave w then sums its
// quarter of the latent dimensions, reading the page a second time, transposed (ds_read_b64_tr_b16: per group of 16 lanes,
// four tokens x 16 dimensions, lane i receives dimension i).
// f32: one workgroup a query row, plain f32 arithmetic.
// A sink takes part in the denominator only, once, when the sums are final.
#include "packed_gemm.hpp"

namespace {

constexpr int kPage = M40LLM_PAGE_TOKENS;

struct LatentArgs {
    const void* queries;
    const void* cache;
    const float* sink;
    const uint32_t *row_slot, *row_pos, *page_table, *tiles;
    void* out;
    float* partial_o;      // [splits][n_queries][latent_pad]
    float* partial_ml;     // [splits][n_queries][2]
    float scale;
    uint32_t heads, latent_pad, k_tiles, max_pages, splits, first_query, n_queries;
};

// sums o of weight l under maximum m, with the sink joined: what o is multiplied by
__device__ __forceinline__ float sink_factor(float m, float l, float sink) {
    const float top = fmaxf(m, sink);
    const float f = expf(m - top);
    return f / fmaf(l, f, expf(sink - top));
}

__device__ __forceinline__ m40_bf16x8 read_transposed(const uint8_t* p0, const uint8_t* p1) {
    typedef short s16x4 __attribute__((ext_vector_type(4)));
    typedef __attribute__((address_space(3))) s16x4* lds4_t;
    typedef short s16x8 __attribute__((ext_vector_type(8)));
    const s16x4 a = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds4_t)(p0));
    const s16x4 b = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds4_t)(p1));
    return __builtin_bit_cast(m40_bf16x8, s16x8{a.x, a.y, a.z, a.w, b.x, b.y, b.z, b.w});
}

template <int MT, int VTW>
__global__ __launch_bounds__(256, 1) void latent_attention_kernel(LatentArgs a) {
    typedef __attribute__((address_space(3))) void* lds_dst_t;
    typedef const __attribute__((address_space(1))) void* global_src_t;
    extern __shared__ __align__(16) uint8_t lds[];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int kt = (int)a.k_tiles;
    uint8_t* q_lds = lds;                                    // [MT][kt] operand tiles
    uint8_t* page_lds = q_lds + MT * kt * 1024;              // [4][kt]
    uint8_t* p_lds = page_lds + 4 * kt * 1024;               // [MT][2]
    float* max_lds = reinterpret_cast<float*>(p_lds + MT * 2048);   // [4][16 MT]
    const uint32_t q0 = a.tiles[2 * blockIdx.x], count = a.tiles[2 * blockIdx.x + 1];
    const uint32_t width = (uint32_t)kt * 32u;
    // the tile's query rows, in operand order
    const m40_bf16* queries = static_cast<const m40_bf16*>(a.queries);
    for (int i = wave; i < MT * kt; i += 4) {
        const int m = i / kt, k = i - m * kt;
        uint32_t r = (uint32_t)(m * 16 + (lane & 15));
        r = r < count ? r : count - 1u;
        *reinterpret_cast<uint4*>(q_lds + i * 1024 + lane * 16) =
            *reinterpret_cast<const uint4*>(queries + (size_t)(q0 + r) * width + k * 32 + (lane >> 4) * 8);
    }
    // positions of the rows this lane holds in result layout; rows past the tile see what its last row sees
    uint32_t pos[MT][4];
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const uint32_t i = (uint32_t)(m * 16 + 4 * (lane >> 4) + r);
            pos[m][r] = a.row_pos[(q0 + (i < count ? i : count - 1u)) / a.heads];
        }
    const uint32_t last_row = (q0 + count - 1u) / a.heads;
    const uint32_t pages = a.row_pos[last_row] / kPage + 1u;
    const uint32_t per_split = (pages + a.splits - 1u) / a.splits;
    const uint32_t page0 = blockIdx.y * per_split, page1 = page0 + per_split < pages ? page0 + per_split : pages;
    const uint32_t* table = a.page_table + (size_t)a.row_slot[last_row] * a.max_pages;
    const m40_bf16* cache = static_cast<const m40_bf16*>(a.cache);
    m40_float4 o[MT][VTW];
    float mx[MT][4], ls[MT][4];
#pragma unroll
    for (int m = 0; m < MT; ++m) {
#pragma unroll
        for (int j = 0; j < VTW; ++j) o[m][j] = m40_float4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int r = 0; r < 4; ++r) { mx[m][r] = -INFINITY; ls[m][r] = 0.0f; }
    }
    const int v_tiles = (int)a.latent_pad / 16;
    for (uint32_t p = page0; p < page1; ++p) {
        const m40_bf16* src = cache + (size_t)table[p] * kPage * width + lane * 8;
        __syncthreads();                                     // the page before has been read (and, first, the queries written)
        for (int i = wave; i < 4 * kt; i += 4)
            __builtin_amdgcn_global_load_lds((global_src_t)(src + (size_t)i * kM40Tile), (lds_dst_t)(page_lds + i * 1024), 16, 0, 0);
        __syncthreads();
        m40_float4 s[MT];
#pragma unroll
        for (int m = 0; m < MT; ++m) s[m] = m40_float4{0.f, 0.f, 0.f, 0.f};
        for (int k = 0; k < kt; ++k) {
            const m40_bf16x8 kf = *reinterpret_cast<const m40_bf16x8*>(page_lds + (wave * kt + k) * 1024 + lane * 16);
#pragma unroll
            for (int m = 0; m < MT; ++m) {
                const m40_bf16x8 qf = *reinterpret_cast<const m40_bf16x8*>(q_lds + (m * kt + k) * 1024 + lane * 16);
                s[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf, kf, s[m], 0, 0, 0);
            }
        }
        const uint32_t key = p * kPage + wave * 16 + (lane & 15);
#pragma unroll
        for (int m = 0; m < MT; ++m)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                s[m][r] = key <= pos[m][r] ? s[m][r] * a.scale : -INFINITY;
                const float t = m40_max16(s[m][r]);
                if ((lane & 15) == 0) max_lds[wave * 16 * MT + m * 16 + 4 * (lane >> 4) + r] = t;
            }
        __syncthreads();
        float alpha[MT][4];
#pragma unroll
        for (int m = 0; m < MT; ++m)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int i = m * 16 + 4 * (lane >> 4) + r;
                float top = mx[m][r];
#pragma unroll
                for (int w = 0; w < 4; ++w) top = fmaxf(top, max_lds[w * 16 * MT + i]);
                const float safe = top == -INFINITY ? 0.0f : top;       // a row that has seen nothing yet
                alpha[m][r] = expf(mx[m][r] - safe);
                mx[m][r] = top;
                const float e = expf(s[m][r] - safe);
                ls[m][r] = ls[m][r] * alpha[m][r] + e;
                // weight of (row i, token 16 wave + lane % 16) in operand order
                const int k = (wave & 1) * 16 + (lane & 15);
                reinterpret_cast<m40_bf16*>(p_lds)[(m * 2 + (wave >> 1)) * kM40Tile + ((k >> 3) * 16 + (i & 15)) * 8 + (k & 7)] = static_cast<m40_bf16>(e);
            }
        __syncthreads();
#pragma unroll
        for (int m = 0; m < MT; ++m)
#pragma unroll
            for (int j = 0; j < VTW; ++j)
#pragma unroll
                for (int r = 0; r < 4; ++r) o[m][j][r] *= alpha[m][r];
        const int g = lane >> 4, li = lane & 15;
#pragma unroll
        for (int c = 0; c < 2; ++c) {
            m40_bf16x8 pf[MT];
#pragma unroll
            for (int m = 0; m < MT; ++m) pf[m] = *reinterpret_cast<const m40_bf16x8*>(p_lds + (m * 2 + c) * 1024 + lane * 16);
            const uint8_t* group = page_lds + (2 * c + (g >> 1)) * kt * 1024;
            const int tok = (g & 1) * 8 + (li >> 2);
#pragma unroll
            for (int j = 0; j < VTW; ++j) {
                const int n = wave * VTW + j;
                if (n < v_tiles) {
                    const int d = n * 16 + (li & 3) * 4;
                    const uint8_t* at = group + (d >> 5) * 1024 + (((d & 31) >> 3) * 16 + tok) * 16 + (d & 7) * 2;
                    const m40_bf16x8 vf = read_transposed(at, at + 4 * 16);
#pragma unroll
                    for (int m = 0; m < MT; ++m) o[m][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pf[m], vf, o[m][j], 0, 0, 0);
                }
            }
        }
    }
    // row sums over the waves
    __syncthreads();
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const float t = m40_sum16(ls[m][r]);
            if ((lane & 15) == 0) max_lds[wave * 16 * MT + m * 16 + 4 * (lane >> 4) + r] = t;
        }
    __syncthreads();
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const uint32_t i = (uint32_t)(m * 16 + 4 * (lane >> 4) + r);
            if (i >= count) continue;
            float l = 0.0f;
#pragma unroll
            for (int w = 0; w < 4; ++w) l += max_lds[w * 16 * MT + i];
            const uint32_t q = q0 + i;
            if (a.splits == 1u) {
                const float f = sink_factor(mx[m][r], l, a.sink[q % a.heads]);
                m40_bf16* out = static_cast<m40_bf16*>(a.out);
                const uint32_t row = q / a.heads, col = q % a.heads * a.latent_pad + (lane & 15);
#pragma unroll
                for (int j = 0; j < VTW; ++j) {
                    const int n = wave * VTW + j;
                    if (n < v_tiles) out[m40_packed_at(row, col + n * 16, a.heads * a.latent_pad / 32u)] = static_cast<m40_bf16>(o[m][j][r] * f);
                }
            } else {
                const size_t at = (size_t)blockIdx.y * a.n_queries + (q - a.first_query);
#pragma unroll
                for (int j = 0; j < VTW; ++j) {
                    const int n = wave * VTW + j;
                    if (n < v_tiles) a.partial_o[at * a.latent_pad + n * 16 + (lane & 15)] = o[m][j][r];
                }
                if (wave == 0 && (lane & 15) == 0) {
                    a.partial_ml[2 * at] = mx[m][r];
                    a.partial_ml[2 * at + 1] = l;
                }
            }
        }
}

// The same walk for up to two row tiles with the query operands in registers and two page buffers: a page is on its way while the
// page before is worked on.  Wave w sums latent column tiles w, w + 4, ...  Tiles past the entry's are read again and multiplied by
// zero, columns past the latent's summed and not stored: a branch around either would put an LDS round trip between products.
// Scores and maxima carry a factor log2(e).
template <int MT, int VTW, int KT>
__global__ __launch_bounds__(256, 1) void latent_decode_kernel(LatentArgs a) {
    typedef __attribute__((address_space(3))) void* lds_dst_t;
    typedef const __attribute__((address_space(1))) void* global_src_t;
    extern __shared__ __align__(16) uint8_t lds[];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int kt = (int)a.k_tiles;
    uint8_t* p_lds = lds + 8 * kt * 1024;                            // behind two pages of [4][kt] tiles: [MT][2]
    float* max_lds = reinterpret_cast<float*>(p_lds + MT * 2048);    // [4][16 MT]
    const uint32_t q0 = a.tiles[2 * blockIdx.x], count = a.tiles[2 * blockIdx.x + 1];
    const uint32_t width = (uint32_t)kt * 32u;
    const uint32_t last_row = (q0 + count - 1u) / a.heads;
    const uint32_t pages = a.row_pos[last_row] / kPage + 1u;
    const uint32_t per_split = (pages + a.splits - 1u) / a.splits;
    const uint32_t page0 = blockIdx.y * per_split, page1 = page0 + per_split < pages ? page0 + per_split : pages;
    const uint32_t* table = a.page_table + (size_t)a.row_slot[last_row] * a.max_pages;
    const m40_bf16* cache = static_cast<const m40_bf16*>(a.cache);
    auto issue = [&](int buf, uint32_t page) __attribute__((always_inline)) {
        const m40_bf16* src = cache + (size_t)page * kPage * width + lane * 8;
        for (int i = wave; i < 4 * kt; i += 4)
            __builtin_amdgcn_global_load_lds((global_src_t)(src + (size_t)i * kM40Tile), (lds_dst_t)(lds + (buf * 4 * kt + i) * 1024), 16, 0, 0);
    };
    uint32_t next_page = 0;
    if (page0 < page1) {
        issue(0, table[page0]);
        next_page = table[page0 + 1 < page1 ? page0 + 1 : page0];
    }
    m40_bf16x8 qf[MT][KT];
    uint32_t pos[MT][4];
#pragma unroll
    for (int m = 0; m < MT; ++m) {
        uint32_t r = (uint32_t)(m * 16 + (lane & 15));
        r = r < count ? r : count - 1u;
        const m40_bf16* src = static_cast<const m40_bf16*>(a.queries) + (size_t)(q0 + r) * width + (lane >> 4) * 8;
#pragma unroll
        for (int k = 0; k < KT; ++k) {
            qf[m][k] = *reinterpret_cast<const m40_bf16x8*>(src + (k < kt ? k : kt - 1) * 32);
            if (k >= kt) qf[m][k] = m40_bf16x8{};
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const uint32_t row = (uint32_t)(m * 16 + 4 * (lane >> 4) + i);
            pos[m][i] = a.row_pos[(q0 + (row < count ? row : count - 1u)) / a.heads];
        }
    }
    m40_float4 o[MT][VTW];
    float mx[MT][4], ls[MT][4];
#pragma unroll
    for (int m = 0; m < MT; ++m) {
#pragma unroll
        for (int j = 0; j < VTW; ++j) o[m][j] = m40_float4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int r = 0; r < 4; ++r) { mx[m][r] = -INFINITY; ls[m][r] = 0.0f; }
    }
    const int v_tiles = (int)a.latent_pad / 16;
    const float scale = a.scale * 1.4426950408889634f;
    int buf = 0;
    for (uint32_t p = page0; p < page1; ++p, buf ^= 1) {
        m40_wait_and_meet<0>();              // page p has landed, and nobody reads the other buffer any more
        if (p + 1 < page1) {
            issue(buf ^ 1, next_page);
            next_page = table[p + 2 < page1 ? p + 2 : p + 1];
        }
        const uint8_t* page_lds = lds + buf * 4 * kt * 1024;
        m40_float4 s[MT];
#pragma unroll
        for (int m = 0; m < MT; ++m) s[m] = m40_float4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int k = 0; k < KT; ++k) {
            const m40_bf16x8 kf = *reinterpret_cast<const m40_bf16x8*>(page_lds + (wave * kt + (k < kt ? k : kt - 1)) * 1024 + lane * 16);
#pragma unroll
            for (int m = 0; m < MT; ++m) s[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf[m][k], kf, s[m], 0, 0, 0);
        }
        const uint32_t key = p * kPage + wave * 16 + (lane & 15);
#pragma unroll
        for (int m = 0; m < MT; ++m)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                s[m][r] = key <= pos[m][r] ? s[m][r] * scale : -INFINITY;
                const float t = m40_max16(s[m][r]);
                if ((lane & 15) == 0) max_lds[wave * 16 * MT + m * 16 + 4 * (lane >> 4) + r] = t;
            }
        m40_wait_and_meet<63>();
        float alpha[MT][4];
#pragma unroll
        for (int m = 0; m < MT; ++m)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int i = m * 16 + 4 * (lane >> 4) + r;
                float top = mx[m][r];
#pragma unroll
                for (int w = 0; w < 4; ++w) top = fmaxf(top, max_lds[w * 16 * MT + i]);
                const float safe = top == -INFINITY ? 0.0f : top;       // a row that has seen nothing yet
                alpha[m][r] = __builtin_amdgcn_exp2f(mx[m][r] - safe);
                mx[m][r] = top;
                const float e = __builtin_amdgcn_exp2f(s[m][r] - safe);
                ls[m][r] = ls[m][r] * alpha[m][r] + e;
                const int k = (wave & 1) * 16 + (lane & 15);
                reinterpret_cast<m40_bf16*>(p_lds)[(m * 2 + (wave >> 1)) * kM40Tile + ((k >> 3) * 16 + (i & 15)) * 8 + (k & 7)] = static_cast<m40_bf16>(e);
            }
        m40_wait_and_meet<63>();
#pragma unroll
        for (int m = 0; m < MT; ++m)
#pragma unroll
            for (int j = 0; j < VTW; ++j)
#pragma unroll
                for (int r = 0; r < 4; ++r) o[m][j][r] *= alpha[m][r];
        const int g = lane >> 4, li = lane & 15, tok = (g & 1) * 8 + (li >> 2);
#pragma unroll
        for (int c = 0; c < 2; ++c) {
            m40_bf16x8 pf[MT];
#pragma unroll
            for (int m = 0; m < MT; ++m) pf[m] = *reinterpret_cast<const m40_bf16x8*>(p_lds + (m * 2 + c) * 1024 + lane * 16);
            const uint8_t* group = page_lds + (2 * c + (g >> 1)) * kt * 1024;
#pragma unroll
            for (int j = 0; j < VTW; ++j) {
                const int n = j * 4 + wave < v_tiles ? j * 4 + wave : v_tiles - 1;
                const int d = n * 16 + (li & 3) * 4;
                const uint8_t* at = group + (d >> 5) * 1024 + (((d & 31) >> 3) * 16 + tok) * 16 + (d & 7) * 2;
                const m40_bf16x8 vf = read_transposed(at, at + 4 * 16);
#pragma unroll
                for (int m = 0; m < MT; ++m) o[m][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pf[m], vf, o[m][j], 0, 0, 0);
            }
        }
    }
    m40_wait_and_meet<0>();
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const float t = m40_sum16(ls[m][r]);
            if ((lane & 15) == 0) max_lds[wave * 16 * MT + m * 16 + 4 * (lane >> 4) + r] = t;
        }
    m40_wait_and_meet<63>();
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const uint32_t i = (uint32_t)(m * 16 + 4 * (lane >> 4) + r);
            if (i >= count) continue;
            float l = 0.0f;
#pragma unroll
            for (int w = 0; w < 4; ++w) l += max_lds[w * 16 * MT + i];
            const uint32_t q = q0 + i;
            mx[m][r] *= 0.6931471805599453f;
            const float f = a.splits == 1u ? sink_factor(mx[m][r], l, a.sink[q % a.heads]) : 1.0f;
            const uint32_t row = q / a.heads, col = q % a.heads * a.latent_pad + (lane & 15);
            const size_t at = (size_t)blockIdx.y * a.n_queries + (q - a.first_query);
#pragma unroll
            for (int j = 0; j < VTW; ++j) {
                const int n = j * 4 + wave;
                if (n >= v_tiles) continue;
                if (a.splits == 1u) static_cast<m40_bf16*>(a.out)[m40_packed_at(row, col + n * 16, a.heads * a.latent_pad / 32u)] = static_cast<m40_bf16>(o[m][j][r] * f);
                else a.partial_o[at * a.latent_pad + n * 16 + (lane & 15)] = o[m][j][r];
            }
            if (a.splits > 1u && wave == 0 && (lane & 15) == 0) {
                a.partial_ml[2 * at] = mx[m][r];
                a.partial_ml[2 * at + 1] = l;
            }
        }
}

__global__ __launch_bounds__(256) void latent_attention_f32_kernel(LatentArgs a) {
    extern __shared__ __align__(16) float flds[];
    float* ql = flds;                        // the query row
    float* ol = ql + a.k_tiles * 32u;        // sums so far
    float* sl = ol + a.latent_pad;           // scores / weights of a page
    __shared__ float stat[3];                // maximum, sum, factor on what came before
    const uint32_t tid = threadIdx.x, q = a.first_query + blockIdx.x, row = q / a.heads, width = a.k_tiles * 32u;
    for (uint32_t i = tid; i < width; i += 256u) ql[i] = static_cast<const float*>(a.queries)[(size_t)q * width + i];
    for (uint32_t i = tid; i < a.latent_pad; i += 256u) ol[i] = 0.0f;
    if (tid == 0) { stat[0] = -INFINITY; stat[1] = 0.0f; }
    const uint32_t pos = a.row_pos[row], pages = pos / kPage + 1u;
    const uint32_t per_split = (pages + a.splits - 1u) / a.splits;
    const uint32_t page0 = blockIdx.y * per_split, page1 = page0 + per_split < pages ? page0 + per_split : pages;
    const uint32_t* table = a.page_table + (size_t)a.row_slot[row] * a.max_pages;
    __syncthreads();
    for (uint32_t p = page0; p < page1; ++p) {
        const float* page = static_cast<const float*>(a.cache) + (size_t)table[p] * kPage * width;
        // four lanes a token, each every fourth group of eight dimensions
        const uint32_t t = tid >> 2, part = tid & 3u;
        const float* entry = page + (size_t)(t / 16u) * a.k_tiles * kM40Tile + (t % 16u) * 8u;
        float s = 0.0f;
        for (uint32_t k8 = part; k8 < width / 8u; k8 += 4u) {
            const float* e = entry + (size_t)(k8 / 4u) * kM40Tile + (k8 % 4u) * 128u;
#pragma unroll
            for (int j = 0; j < 8; ++j) s = fmaf(ql[k8 * 8u + j], e[j], s);
        }
        s += m40_dpp_f<M40_DPP_XOR1>(s);
        s += m40_dpp_f<M40_DPP_XOR2>(s);
        if (part == 0u) sl[t] = p * kPage + t <= pos ? s * a.scale : -INFINITY;
        __syncthreads();
        if (tid < 64u) {
            const float v = sl[tid], before = stat[0], top = fmaxf(before, m40_max64(v));   // a page of the range holds a seen token
            const float e = expf(v - top), f = expf(before - top), sum = m40_sum64(e);
            sl[tid] = e;
            if (tid == 0u) { stat[0] = top; stat[1] = stat[1] * f + sum; stat[2] = f; }
        }
        __syncthreads();
        const float f = stat[2];
        for (uint32_t d = tid; d < a.latent_pad; d += 256u) {
            float acc = ol[d] * f;
            const float* col = page + (size_t)(d / 32u) * kM40Tile + m40_tile_offset(0, d % 32u);
            for (uint32_t t2 = 0; t2 < (uint32_t)kPage; ++t2) acc = fmaf(sl[t2], col[(size_t)(t2 / 16u) * a.k_tiles * kM40Tile + (t2 % 16u) * 8u], acc);
            ol[d] = acc;
        }
        __syncthreads();
    }
    const float m = stat[0], l = stat[1];
    if (a.splits == 1u) {
        const float f = sink_factor(m, l, a.sink[q % a.heads]);
        for (uint32_t d = tid; d < a.latent_pad; d += 256u) static_cast<float*>(a.out)[m40_packed_at(row, q % a.heads * a.latent_pad + d, a.heads * a.latent_pad / 32u)] = ol[d] * f;
    } else {
        const size_t at = (size_t)blockIdx.y * a.n_queries + blockIdx.x;
        for (uint32_t d = tid; d < a.latent_pad; d += 256u) a.partial_o[at * a.latent_pad + d] = ol[d];
        if (tid == 0u) { a.partial_ml[2 * at] = m; a.partial_ml[2 * at + 1] = l; }
    }
}

// Joins the splits of a query row with its sink: a workgroup takes 128 dimensions of one row, eight groups of 32 lanes every
// eighth split each.
constexpr int kJoinSplits = 512;
template <class T>
__global__ __launch_bounds__(256) void latent_attention_join_kernel(LatentArgs a) {
    __shared__ float weight[kJoinSplits];
    __shared__ m40_float4 sums[8][32];
    __shared__ float part[4], den_part[4];
    const uint32_t i = blockIdx.x, q = a.first_query + i, tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6;
    const float sink = a.sink[q % a.heads];
    const float2* ml = reinterpret_cast<const float2*>(a.partial_ml);
    float2 mine[kJoinSplits / 256];
    float top = sink;
#pragma unroll
    for (int j = 0; j < kJoinSplits / 256; ++j) {
        const uint32_t s = tid + 256u * j;
        mine[j] = s < a.splits ? ml[(size_t)s * a.n_queries + i] : make_float2(-INFINITY, 0.0f);
        top = fmaxf(top, mine[j].x);
    }
    top = m40_max64(top);
    if (lane == 0) part[wave] = top;
    __syncthreads();
    top = fmaxf(fmaxf(part[0], part[1]), fmaxf(part[2], part[3]));
    float den = 0.0f;
#pragma unroll
    for (int j = 0; j < kJoinSplits / 256; ++j) {
        const uint32_t s = tid + 256u * j;
        const float e = expf(mine[j].x - top);
        if (s < a.splits) weight[s] = e;
        den = fmaf(mine[j].y, e, den);
    }
    den = m40_sum64(den);
    if (lane == 0) den_part[wave] = den;
    __syncthreads();
    const float inv = 1.0f / (den_part[0] + den_part[1] + den_part[2] + den_part[3] + expf(sink - top));
    const uint32_t d = blockIdx.y * 128u + (tid & 31u) * 4u, group = tid >> 5;
    m40_float4 acc = {0.f, 0.f, 0.f, 0.f};
    if (d < a.latent_pad) {
        const float* o = a.partial_o + (size_t)i * a.latent_pad + d;
        const size_t stride = (size_t)a.n_queries * a.latent_pad;
#pragma unroll 4
        for (uint32_t s = group; s < a.splits; s += 8u) acc += *reinterpret_cast<const m40_float4*>(o + s * stride) * weight[s];
    }
    sums[group][tid & 31u] = acc;
    __syncthreads();
    if (group != 0 || d >= a.latent_pad) return;
#pragma unroll
    for (int g = 1; g < 8; ++g) acc += sums[g][tid & 31u];
    m40_store4<T>(static_cast<T*>(a.out) + m40_packed_at(q / a.heads, q % a.heads * a.latent_pad + d, a.heads * a.latent_pad / 32u), acc * inv);
}

constexpr int kLdsMax = 160 * 1024;
int lds_bytes(int mt, int k_tiles) { return (mt + 4) * k_tiles * 1024 + mt * 2048 + 4 * 16 * mt * 4; }

template <int MT, int VTW>
int launch_bf16(hipStream_t stream, const LatentArgs& a, uint32_t n_tiles) {
    static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(latent_attention_kernel<MT, VTW>),
                                                       hipFuncAttributeMaxDynamicSharedMemorySize, kLdsMax);
    if (attr != hipSuccess) return -2;
    latent_attention_kernel<MT, VTW><<<dim3(n_tiles, a.splits), 256, lds_bytes(MT, (int)a.k_tiles), stream>>>(a);
    return hipGetLastError() == hipSuccess ? 0 : -2;
}
template <int MT, int VTW, int KT>
int launch_decode(hipStream_t stream, const LatentArgs& a, uint32_t n_tiles) {
    static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(latent_decode_kernel<MT, VTW, KT>),
                                                       hipFuncAttributeMaxDynamicSharedMemorySize, kLdsMax);
    if (attr != hipSuccess) return -2;
    latent_decode_kernel<MT, VTW, KT><<<dim3(n_tiles, a.splits), 256, (int)a.k_tiles * 8 * 1024 + MT * 2048 + 4 * 16 * MT * 4, stream>>>(a);
    return hipGetLastError() == hipSuccess ? 0 : -2;
}
template <int MT>
int launch_bf16_m(hipStream_t stream, const LatentArgs& a, uint32_t n_tiles) {
    const uint32_t per_wave = (a.latent_pad / 16u + 3u) / 4u;
    if constexpr (MT <= 2) {
        if (a.k_tiles <= 6u && per_wave <= 3u) return launch_decode<MT, 3, 6>(stream, a, n_tiles);
        if (a.k_tiles <= 10u && per_wave <= 4u) return launch_decode<MT, 4, 10>(stream, a, n_tiles);
        if (a.k_tiles <= 18u && per_wave <= 8u) return launch_decode<MT, 8, 18>(stream, a, n_tiles);
        if (a.k_tiles <= 19u && per_wave <= 10u) return launch_decode<MT, 10, 19>(stream, a, n_tiles);
    }
    if (per_wave <= 1u) return launch_bf16<MT, 1>(stream, a, n_tiles);
    if (per_wave <= 2u) return launch_bf16<MT, 2>(stream, a, n_tiles);
    if (per_wave <= 4u) return launch_bf16<MT, 4>(stream, a, n_tiles);
    if (per_wave <= 8u) return launch_bf16<MT, 8>(stream, a, n_tiles);
    if constexpr (MT <= 2) {
        if (per_wave <= 16u) return launch_bf16<MT, 16>(stream, a, n_tiles);
    }
    return -3;
}

}  // namespace

extern "C" {

uint64_t m40llm_ext_latent_attention_partial_floats(uint32_t n_queries, uint32_t latent_pad, uint32_t splits) {
    return splits <= 1u ? 0u : (uint64_t)splits * n_queries * (latent_pad + 2u);
}

uint32_t m40llm_ext_latent_attention_max_m_tiles(uint32_t act_dtype, uint32_t kv_rank, uint32_t entry_width) {
    const uint32_t latent_pad = (kv_rank + 31u) / 32u * 32u;
    if (act_dtype == M40LLM_ACT_F32) return (entry_width + latent_pad + kPage) * 4u <= 60u * 1024u ? 4u : 0u;
    for (uint32_t mt = 4; mt >= 1; mt /= 2)
        if (lds_bytes((int)mt, (int)entry_width / 32) <= kLdsMax && (latent_pad / 16u + 3u) / 4u <= (mt <= 2 ? 16u : 8u)) return mt;
    return 0;
}

int m40llm_ext_latent_attention_async(M40llmCudaContext* ctx, const M40llmLatentAttention* p, uint32_t stream_kind) {
    if (!ctx || !p || !p->queries || !p->cache || !p->sink || !p->row_slot || !p->row_pos || !p->page_table || !p->tiles || !p->out) return -1;
    hipStream_t stream = m40_select_stream(ctx, stream_kind);
    if (!stream || m40_ensure_device(ctx) != 0) return -2;
    if (p->act_dtype > 1u || p->heads == 0 || p->kv_rank == 0 || p->latent_pad != (p->kv_rank + 31u) / 32u * 32u ||
        p->entry_width % 32u != 0 || p->entry_width < p->latent_pad || p->n_tiles == 0 || p->splits == 0 || p->splits > (uint32_t)kJoinSplits ||
        p->n_queries == 0)
        return -3;
    const uint32_t max_mt = m40llm_ext_latent_attention_max_m_tiles(p->act_dtype, p->kv_rank, p->entry_width);
    if (p->m_tiles == 0 || p->m_tiles > max_mt) return -3;
    LatentArgs a{};
    a.queries = p->queries; a.cache = p->cache; a.sink = static_cast<const float*>(p->sink);
    a.row_slot = p->row_slot; a.row_pos = p->row_pos; a.page_table = p->page_table; a.tiles = p->tiles;
    a.out = p->out; a.scale = p->scale; a.heads = p->heads; a.latent_pad = p->latent_pad; a.k_tiles = p->entry_width / 32u;
    a.max_pages = p->max_pages; a.splits = p->splits; a.first_query = p->first_query; a.n_queries = p->n_queries;
    if (p->splits > 1u) {
        if (!p->partial || p->partial_floats < m40llm_ext_latent_attention_partial_floats(p->n_queries, p->latent_pad, p->splits)) return -4;
        a.partial_o = static_cast<float*>(p->partial);
        a.partial_ml = a.partial_o + (size_t)p->splits * p->n_queries * p->latent_pad;
    }
    (void)hipGetLastError();
    int rc = -3;
    if (p->act_dtype == M40LLM_ACT_F32) {
        latent_attention_f32_kernel<<<dim3(p->n_queries, p->splits), 256, (p->entry_width + p->latent_pad + kPage) * 4u, stream>>>(a);
        rc = hipGetLastError() == hipSuccess ? 0 : -2;
    } else if (p->m_tiles == 1u) rc = launch_bf16_m<1>(stream, a, p->n_tiles);
    else if (p->m_tiles == 2u) rc = launch_bf16_m<2>(stream, a, p->n_tiles);
    else rc = launch_bf16_m<4>(stream, a, p->n_tiles);
    if (rc != 0 || p->splits == 1u) return rc;
    const dim3 join(p->n_queries, (p->latent_pad + 127u) / 128u);
    if (p->act_dtype == M40LLM_ACT_F32) latent_attention_join_kernel<float><<<join, 256, 0, stream>>>(a);
    else latent_attention_join_kernel<m40_bf16><<<join, 256, 0, stream>>>(a);
    return hipGetLastError() == hipSuccess ? 0 : -2;
}

}  // extern "C"
