// What the layers of a decoder share: the pass they run (rows, portions, device tables), the residual stream and the scratch buffers,
// packing of weights, and launches of packed products.
#pragma once

#include <algorithm>
#include <cstring>
#include <functional>
#include <memory>
#include <string>
#include <vector>

#include "decoder_spec.hpp"
#include "model.hpp"
#include "page_pool.hpp"
#include "safetensors.hpp"

namespace m40host {

inline uint32_t round_up(uint32_t n, uint32_t m) { return (n + m - 1) / m * m; }

struct LayeredOptions {
    uint32_t act_dtype = M40LLM_ACT_BF16;
    uint32_t max_tokens = 4096;        // what the cache pool holds, in tokens
    uint32_t max_sequences = 4;
    uint32_t max_rows = 4096;          // rows of one pass; longer steps run in several
    uint32_t portion_form = 0;         // attention of portions: 0 the cheaper form, 1 that of single tokens, 2 that of long portions where it is served
};

struct Portion { uint32_t row, n, slot, length; bool is_long; };      // length: tokens its sequence holds at its end
struct PassPlan {
    std::vector<uint32_t> tokens, prev, slot, pos, back, want;
    std::vector<size_t> want_out;
    std::vector<Portion> portions;
    uint32_t short_rows = 0;           // rows before it belong to single tokens and short portions, from it on to long portions
    uint32_t rows() const { return (uint32_t)tokens.size(); }
};
// device addresses of a pass
struct Rows {
    uint32_t rows = 0, short_rows = 0;
    bool in_place = false;             // every layer leaves its result in x
    uint32_t *tokens = nullptr, *prev = nullptr, *slot = nullptr, *pos = nullptr, *back = nullptr, *page_table = nullptr;
    uint32_t multi_row_portions = 0;   // portions of two rows and more
};

// A table that some layers need beside rows, positions and pages; made anew for every pass.
class PassTable {
public:
    virtual ~PassTable() = default;
    virtual std::vector<uint32_t> build(const PassPlan& plan, const SequencePages& pages, uint32_t longest) = 0;    // longest: most tokens a short portion sees
    virtual uint64_t partial_floats(const Rows&) const { return 0; }
    virtual void enqueue(const Rows&) {}                // what the device makes itself, at the start of a pass
    const uint32_t* at = nullptr;
};

// {first row, rows, slot, 0} of every portion, single rows first, then the 64-row groups of the pass that the others touch
class PortionTable : public PassTable {
public:
    uint32_t n = 0, singles = 0, n_chunks = 0;
    const uint32_t* multi() const { return at + 4 * singles; }
    const uint32_t* chunk_base() const { return at + 4 * n; }
    const uint32_t* chunks() const { return at + 4 * n + (n - singles); }
    std::vector<uint32_t> build(const PassPlan& plan, const SequencePages&, uint32_t) override {
        std::vector<uint32_t> t, base, groups;
        n = (uint32_t)plan.portions.size();
        for (const Portion& p : plan.portions)
            if (p.n == 1) t.insert(t.end(), {p.row, p.n, p.slot, 0u});
        singles = (uint32_t)t.size() / 4;
        uint32_t k = 0;
        for (const Portion& p : plan.portions) {
            if (p.n == 1) continue;
            t.insert(t.end(), {p.row, p.n, p.slot, 0u});
            base.push_back((uint32_t)groups.size() / 2);
            for (uint32_t g = p.row / 64; g <= (p.row + p.n - 1) / 64; ++g) groups.insert(groups.end(), {k, g * 64});
            ++k;
        }
        n_chunks = (uint32_t)groups.size() / 2;
        t.insert(t.end(), base.begin(), base.end());
        t.insert(t.end(), groups.begin(), groups.end());
        return t;
    }
};

// a buffer that layers use one after the other: as large as the largest asks for
struct Scratch {
    DeviceBuf buf;
    size_t bytes = 0;
    void want(size_t n) { bytes = std::max(bytes, n); }
    void* ptr() const { return buf.ptr(); }
    float* f32(size_t off = 0) const { return buf.f32(off); }
    uint32_t* u32(size_t off = 0) const { return buf.u32(off); }
};

struct SlotState { DeviceBuf* buf; size_t slot_bytes; };      // what a layer carries from token to token, per sequence slot

class LayerRuntime {
public:
    static constexpr uint32_t kStream = M40LLM_STREAM_DECODE;
    static constexpr uint32_t kPage = M40LLM_PAGE_TOKENS;
    static constexpr uint32_t kCus = 256, kMaxParts = 8;

    LayerRuntime(M40llmCudaContext* c, const DecoderSpec& s, const LayeredOptions& o, uint32_t pages)
        : ctx(c), spec(s), opt(o), es(o.act_dtype == M40LLM_ACT_F32 ? 4u : 2u), max_pages(pages), d_pad(round_up(s.width, 32)),
          rows_pad(round_up(std::max(o.max_rows, o.max_sequences), 64)) {}

    M40llmCudaContext* ctx;
    const DecoderSpec& spec;
    LayeredOptions opt;
    uint32_t es, max_pages, d_pad, rows_pad;
    uint32_t pending = 0;              // planes whose sums x has not taken yet
    std::vector<std::unique_ptr<PassTable>> tables;
    std::vector<SlotState> states;
    DeviceBuf x, partial;
    Scratch planes, h, h_rows, proj, cat;
    std::vector<Scratch*> scratch{&planes, &h, &h_rows, &proj, &cat};
    uint64_t plane_floats = 4;

    bool bf16() const { return opt.act_dtype == M40LLM_ACT_BF16; }
    size_t act_bytes(size_t cols) const { return (size_t)rows_pad * cols * es; }
    size_t f32_bytes(size_t cols) const { return (size_t)rows_pad * cols * 4; }

    // ---- setting up
    DeviceBuf cleared(size_t bytes) {
        DeviceBuf b(ctx, (bytes + 15) / 16 * 16);
        M40H_TRY(m40llm_ext_clear_u32_async(ctx, b.ptr(), b.bytes() / 4, kStream));
        return b;
    }
    DeviceBuf upload_f32(const std::vector<float>& v) {
        DeviceBuf b(ctx, v.size() * 4);
        M40H_TRY(m40llm_memcpy_h2d(ctx, b.ptr(), v.data(), v.size() * 4));
        return b;
    }
    DeviceBuf upload_norm(TensorSource& t, const std::string& name) {         // of the residual's width
        if (spec.norm_scalar) return upload_f32(std::vector<float>(spec.width, t.read_f32(name, {})[0]));
        std::vector<float> w = t.read_f32(name, {spec.width});
        if (spec.norm_around_zero)
            for (float& x : w) x += 1.0f;
        return upload_f32(w);
    }
    // [columns][taps] to [taps][columns]
    DeviceBuf upload_taps(TensorSource& t, const std::string& name, uint32_t cols, uint32_t taps) {
        const std::vector<float> w = t.read_f32(name, {cols, taps});
        std::vector<float> o(w.size());
        for (uint32_t c = 0; c < cols; ++c)
            for (uint32_t j = 0; j < taps; ++j) o[(size_t)j * cols + c] = w[(size_t)c * taps + j];
        return upload_f32(o);
    }
    void* stage(TensorSource& t, const std::string& name, const std::vector<uint64_t>& shape) {
        const size_t bytes = tensor_elements(shape) * 2;
        M40H_TRY(m40llm_stream_synchronize(ctx, kStream));       // the tensor before may still be being packed
        if (staging_.bytes() < bytes) staging_ = DeviceBuf(ctx, bytes);
        t.read_bf16(ctx, name, shape, staging_.ptr());
        return staging_.ptr();
    }
    DeviceBuf packed(uint32_t n_tiles, uint32_t k_tiles) { return cleared((size_t)n_tiles * k_tiles * 1024); }
    // rows [N][K] of a plain matrix from row / column offsets on
    void pack(TensorSource& t, const std::string& name, uint32_t N, uint32_t K, void* dst, uint32_t k_tiles, uint32_t tile_first,
              uint32_t k_offset = 0, uint32_t tile_stride = 1) {
        pack_rows(stage(t, name, {N, K}), 0, N, K, dst, k_tiles, tile_first, k_offset, tile_stride);
    }
    void pack_rows(const void* src, uint32_t first, uint32_t N, uint32_t K, void* dst, uint32_t k_tiles, uint32_t tile_first, uint32_t k_offset = 0,
                   uint32_t tile_stride = 1) {
        M40llmPackPlan p{};
        p.n_blocks = 1; p.n = N; p.n_block_pad = N;
        p.k_blocks = 1; p.k = K; p.k_block_pad = K; p.k_offset = k_offset;
        p.sn = K; p.sk = 1;
        p.k_tiles = k_tiles; p.tile_first = tile_first; p.tile_stride = tile_stride;
        M40H_TRY(m40llm_ext_pack_tiles_async(ctx, static_cast<const uint16_t*>(src) + (size_t)first * K, dst, &p, kStream));
    }
    // per head: rows [first, first + n) of the head's `stride` rows of [heads * stride][K] to packed rows offset .. of its block_pad, from
    // row tile tile_first on
    void pack_heads(const void* src, uint32_t heads, uint32_t stride, uint32_t first, uint32_t n, uint32_t K, void* dst, uint32_t k_tiles,
                    uint32_t block_pad, uint32_t offset, uint32_t tile_first = 0) {
        M40llmPackPlan p{};
        p.n_blocks = heads; p.n = n; p.n_block_pad = block_pad; p.n_offset = offset;
        p.k_blocks = 1; p.k = K; p.k_block_pad = K;
        p.sn_block = (uint64_t)stride * K; p.sn = K; p.sk = 1;
        p.k_tiles = k_tiles; p.tile_first = tile_first; p.tile_stride = 1;
        M40H_TRY(m40llm_ext_pack_tiles_async(ctx, static_cast<const uint16_t*>(src) + (size_t)first * K, dst, &p, kStream));
    }
    void finish_loading() {
        M40H_TRY(m40llm_stream_synchronize(ctx, kStream));
        staging_ = DeviceBuf();
    }
    // The layers' table of this type and key: made once, shared by all that ask for the same.
    template <class T, class... A>
    T& table(A... args) {
        for (auto& t : tables)
            if (auto* p = dynamic_cast<T*>(t.get()); p && p->same(args...)) return *p;
        tables.push_back(std::make_unique<T>(args...));
        return static_cast<T&>(*tables.back());
    }
    PortionTable& portions() {
        if (!portions_) {
            tables.push_back(std::make_unique<PortionTable>());
            portions_ = static_cast<PortionTable*>(tables.back().get());
        }
        return *portions_;
    }
    void allocate() {
        x = cleared((size_t)rows_pad * spec.width * 4);
        h.want(act_bytes(d_pad));
        planes.want(plane_floats * 4);
        for (Scratch* s : scratch)
            if (s->bytes) s->buf = cleared(s->bytes);
    }

    // ---- launches
    M40llmPackedGemm product(const void* a, uint32_t lda, const DeviceBuf& w, uint32_t n_tiles, uint32_t k_tiles, uint32_t rows, uint32_t epilogue) const {
        M40llmPackedGemm g{};
        g.act_dtype = opt.act_dtype; g.epilogue = epilogue;
        g.a = a; g.lda = lda; g.w = w.ptr(); g.n_tiles = n_tiles; g.k_tiles = k_tiles;
        g.rows = rows; g.batches = 1;
        return g;
    }
    void launch(const M40llmPackedGemm& g) { M40H_TRY(m40llm_ext_packed_gemm_async(ctx, &g, kStream)); }
    char* act(void* b, size_t elements) const { return static_cast<char*>(b) + elements * es; }
    // Into how many parts the sum over a product's k tiles is cut where a launch would leave CUs idle.
    uint32_t k_parts(uint32_t n_tiles, uint32_t k_tiles, uint32_t rows) const {
        uint32_t groups;
        if (rows <= 64 || !bf16()) groups = n_tiles * ((rows + 63) / 64);
        else groups = (rows + 127) / 128 * ((n_tiles + 7) / 8);
        uint32_t parts = 1;
        while (parts < kMaxParts && groups * parts * 2 <= kCus && k_tiles / (parts * 2) >= 32) parts *= 2;
        return (parts - 1) * ((k_tiles + parts - 1) / parts) < k_tiles ? parts : 1u;
    }
    // most floats the planes of a product with `width` columns take at any number of rows
    void want_planes(uint32_t k_tiles, bool whole_too) {
        for (uint32_t rows = 1; rows <= rows_pad; ++rows) {
            const uint32_t parts = k_parts(round_up(spec.width, 16) / 16, k_tiles, rows);
            if (parts > 1 || whole_too) plane_floats = std::max<uint64_t>(plane_floats, (uint64_t)parts * rows * spec.width);
        }
    }
    // a product with `width` columns into planes, which whoever comes next adds up; returns how many
    uint32_t into_planes(M40llmPackedGemm g, uint32_t rows) {
        g.epilogue = M40LLM_PACKED_STORE;
        g.ld_out = spec.width; g.cols = spec.width;
        g.k_parts = k_parts(g.n_tiles, g.k_tiles, rows);
        g.out_f32 = planes.ptr(); g.out_batch = (uint64_t)rows * spec.width;
        launch(g);
        return g.k_parts;
    }

private:
    DeviceBuf staging_;
    PortionTable* portions_ = nullptr;
};

// cosines and sines of a pass's rows
struct RotationAngles : PassTable {
    RotationAngles(LayerRuntime* rt, RotationSpec s, uint32_t h) : rt_(rt), spec(s), half(h) {
        const std::vector<double> f = spec.frequencies();
        freq_ = DeviceBuf(rt->ctx, std::max<size_t>(f.size(), 1) * 8);
        if (!f.empty()) M40H_TRY(m40llm_memcpy_h2d(rt->ctx, freq_.ptr(), f.data(), f.size() * 8));
        angles = rt->cleared((size_t)rt->rows_pad * half * 8);
    }
    bool same(LayerRuntime*, const RotationSpec& s, uint32_t h) const { return spec == s && half == h; }
    std::vector<uint32_t> build(const PassPlan&, const SequencePages&, uint32_t) override { return {}; }
    void enqueue(const Rows& r) override {
        M40H_TRY(m40llm_ext_rotation_angles_async(rt_->ctx, r.pos, r.rows, static_cast<const double*>(freq_.ptr()), spec.dims / 2, half,
                                                  (float)spec.magnitude(), angles.ptr(), LayerRuntime::kStream));
    }
    LayerRuntime* rt_;
    RotationSpec spec;
    uint32_t half;                        // padded pairs of a row
    DeviceBuf freq_, angles;
};

// One layer (or block) of a decoder.
class DecoderLayer {
public:
    virtual ~DecoderLayer() = default;
    virtual void enqueue(const Rows& r) = 0;
    virtual void prepare(const Rows&) {}                 // scratch whose size depends on the pass
    // Work of the attention of a portion of n tokens behind `len`, in flops, as single tokens and as a long portion; false where it has no
    // second form.
    virtual bool portion_cost(uint32_t n, uint32_t len, double& as_tokens, double& as_long) const { (void)n; (void)len; (void)as_tokens; (void)as_long; return true; }
};

}  // namespace m40host
