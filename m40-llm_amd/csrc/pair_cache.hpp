// Pages of a cache of keys and values whose keys come in one or two maps a head (include/m40llm.h has the order).
#pragma once

#include "packed_gemm.hpp"

#define M40LLM_PAIR_MOST_DIM 256u

struct M40PairPage {
    uint32_t maps, kv_heads, k_tiles, v_tiles;
    M40_HD M40PairPage(uint32_t maps_, uint32_t heads, uint32_t dim, uint32_t vdim) : maps(maps_), kv_heads(heads), k_tiles((dim + 31u) / 32u), v_tiles((vdim + 15u) / 16u) {}
    M40_HD size_t key_elements() const { return (size_t)4u * maps * k_tiles * 512u; }                // all maps of a kv head
    M40_HD size_t head_elements() const { return key_elements() + (size_t)2u * v_tiles * 512u; }
    M40_HD size_t elements() const { return kv_heads * head_elements(); }
#ifdef __HIPCC__
    // dimension d of the page's token t
    __device__ __forceinline__ size_t key_at(uint32_t map, uint32_t t, uint32_t d) const {
        return (size_t)((map * 4u + t / 16u) * k_tiles + d / 32u) * kM40Tile + m40_tile_offset(t % 16u, d % 32u);
    }
    __device__ __forceinline__ size_t value_at(uint32_t t, uint32_t d) const {
        const uint32_t in = t % 32u, place = (in % 16u) / 4u * 8u + in / 16u * 4u + in % 4u;
        return key_elements() + (size_t)((d / 16u) * 2u + t / 32u) * kM40Tile + ((place >> 3) * 16u + d % 16u) * 8u + (place & 7u);
    }
#endif
};
