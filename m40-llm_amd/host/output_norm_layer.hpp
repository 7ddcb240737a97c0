// Layers whose sublayers read the residual stream itself and have a norm on their output: x += m * norm1(mixer(x)), then
// x += m * norm2(feed-forward(x)).  A sublayer's last product leaves its sums in planes; one launch adds them up, norms them, adds them to
// x and writes x as the next products' operand.
#pragma once

#include "layer_runtime.hpp"

namespace m40host {

class Mixer {
public:
    virtual ~Mixer() = default;
    virtual uint32_t enqueue(const Rows& r) = 0;         // returns the number of planes
    virtual void prepare(const Rows&) {}
    virtual bool portion_cost(uint32_t, uint32_t, double&, double&) const { return true; }
    virtual bool reads_plain_rows() const { return false; }      // it wants its input as plain rows (h_rows) as well
};

// Tiles of queries (row, head of a kv head's group): 16 a tile for single tokens and short portions, 64 or 128 for long ones.  window: of the
// newest tokens, which is all that queries see (0 = everything).
struct PairTiles : PassTable {
    PairTiles(uint32_t g, uint32_t most, uint32_t w) : group(g), most_queries(most), window(w ? w : 0x7fffffffu) {}
    bool same(uint32_t g, uint32_t most, uint32_t w) const { return group == g && most_queries == most && window == (w ? w : 0x7fffffffu); }
    uint32_t group, most_queries, window, fewest_kv_heads = 0xffffffffu, n_short = 0, n_long = 0, long_queries = 64, splits = 1;
    bool even = false;                    // long tiles see about equally many keys
    uint64_t floats_a_row = 0;            // of a split's partial sums, the largest layer's
    const uint32_t* long_tiles() const { return at + 2 * n_short; }
    std::vector<uint32_t> build(const PassPlan& plan, const SequencePages&, uint32_t longest) override {
        std::vector<uint32_t> t;
        uint64_t blocks = 0;
        for (const Portion& p : plan.portions) {
            const uint32_t n = p.n * group;
            for (uint32_t i = 0; !p.is_long && i < n; i += 16) t.insert(t.end(), {p.row * group + i, std::min(16u, n - i)});
            if (p.is_long) blocks += (n + 127) / 128;
        }
        n_short = (uint32_t)t.size() / 2;
        long_queries = most_queries >= 128 && blocks * fewest_kv_heads >= LayerRuntime::kCus ? 128u : 64u;
        struct Tile { uint32_t first, n, keys; };
        std::vector<Tile> tiles;
        for (const Portion& p : plan.portions) {
            const uint32_t n = p.n * group;
            for (uint32_t i = 0; p.is_long && i < n; i += long_queries) {
                const uint32_t m = std::min(long_queries, n - i);
                const uint32_t first = p.length - p.n + i / group + 1, last = p.length - p.n + (i + m + group - 1) / group;
                tiles.push_back({p.row * group + i, m, last - (first > window ? first - window : 0)});
            }
        }
        std::stable_sort(tiles.begin(), tiles.end(), [](const Tile& a, const Tile& b) { return a.keys > b.keys; });     // the longest walks first
        uint64_t keys = 0;
        for (const Tile& x : tiles) {
            t.insert(t.end(), {x.first, x.n});
            keys += x.keys;
        }
        even = !tiles.empty() && (uint64_t)tiles[0].keys * tiles.size() <= keys + keys / 4;
        n_long = (uint32_t)tiles.size();
        // the pages of a tile over as many workgroups as fill the CUs twice, a page a wave at least
        const uint32_t seen = longest > window ? window + LayerRuntime::kPage : longest;
        const uint32_t pages = (seen + LayerRuntime::kPage - 1) / LayerRuntime::kPage, groups = std::max(1u, n_short * fewest_kv_heads);
        splits = std::max(1u, std::min({(pages + 3) / 4, 2 * LayerRuntime::kCus / groups, 256u}));
        return t;
    }
    uint64_t partial_floats(const Rows& r) const override { return splits <= 1 ? 0 : (uint64_t)splits * r.short_rows * floats_a_row; }
};

struct PairShared { Scratch queries; };       // buffers all differential attention layers of a decoder share

// Launches: product (projections and gate logits) | convolution, norms, cache append | (state of longer portions) | attention | product
class DifferentialMixer : public Mixer {
public:
    DifferentialMixer(LayerRuntime& rt, std::shared_ptr<PairShared> shared, TensorSource& t, uint32_t index, const DifferentialAttentionSpec& a, DifferentialMixer* source)
        : rt_(rt), sh_(std::move(shared)), a_(a), source_(source), portions_(rt.portions()) {
        const std::string p = "l" + std::to_string(index) + ".mix.";
        most_queries_ = m40llm_ext_pair_attention_tile_queries(rt.opt.act_dtype, 2, a.dim, a.vdim);
        if (most_queries_ == 0) throw std::invalid_argument("layer " + std::to_string(index) + ": head sizes beyond what the attention kernels serve");
        const uint32_t q = 2 * a.heads * a.dim, k = 2 * a.kv_heads * a.dim, v = a.kv_heads * a.vdim;
        k_offset_ = round_up(q, 16);
        v_offset_ = k_offset_ + (source ? 0 : round_up(k, 16));
        gate_offset_ = v_offset_ + (source ? 0 : round_up(v, 16));
        conv_cols_ = round_up(source ? q : v_offset_ + v, 4);
        tiles_in_ = round_up(gate_offset_ + a.heads, 16) / 16;
        o_pad_ = round_up(a.heads * a.vdim, 32);
        const uint32_t D = rt.spec.width, d_tiles = rt.d_pad / 32;
        w_in_ = rt.packed(tiles_in_, d_tiles);
        rt.pack(t, p + "q", q, D, w_in_.ptr(), d_tiles, 0);
        std::vector<float> q_norm = t.read_f32(p + "q.norm", {a.dim});
        if (a.scale < 0.0f)                   // the kernels take the scale's sign from the queries
            for (float& w : q_norm) w = -w;
        q_norm_ = rt.upload_f32(q_norm);
        if (a.taps) q_conv_ = rt.upload_taps(t, p + "q.conv", q, a.taps);
        if (!source) {
            rt.pack(t, p + "k", k, D, w_in_.ptr(), d_tiles, k_offset_ / 16);
            rt.pack(t, p + "v", v, D, w_in_.ptr(), d_tiles, v_offset_ / 16);
            k_norm_ = rt.upload_f32(t.read_f32(p + "k.norm", {a.dim}));
            if (a.taps) {
                k_conv_ = rt.upload_taps(t, p + "k.conv", k, a.taps);
                v_conv_ = rt.upload_taps(t, p + "v.conv", v, a.taps);
            }
            cache_ = rt.cleared((size_t)rt.max_pages * m40llm_ext_pair_page_elements(2, a.kv_heads, a.dim, a.vdim) * rt.es);
        }
        rt.pack(t, p + "g", a.heads, D, w_in_.ptr(), d_tiles, gate_offset_ / 16);
        w_out_ = rt.packed(round_up(D, 16) / 16, o_pad_ / 32);
        rt.pack(t, p + "o", D, a.heads * a.vdim, w_out_.ptr(), o_pad_ / 32, 0);
        auto dot = [&](const char* x, const char* y) {
            const std::vector<float> u = t.read_f32(p + x, {a.dim}), w = t.read_f32(p + y, {a.dim});
            double s = 0.0;
            for (uint32_t i = 0; i < a.dim; ++i) s += (double)u[i] * w[i];
            return s;
        };
        lambda_ = (float)(std::exp(dot("lq1", "lk1")) - std::exp(dot("lq2", "lk2")) + a.diff);
        if (a.taps > 1) {
            const size_t slot = (size_t)(a.taps - 1) * conv_cols_ * 4;
            conv_state_ = rt.cleared(slot * rt.opt.max_sequences);
            rt.states.push_back({&conv_state_, slot});
        }
        tiles_ = &rt.table<PairTiles>(a.heads / a.kv_heads, most_queries_, 0u);
        tiles_->fewest_kv_heads = std::min(tiles_->fewest_kv_heads, a.kv_heads);
        tiles_->floats_a_row = std::max(tiles_->floats_a_row, m40llm_ext_pair_attention_partial_floats(2, 1, a.heads, a.vdim, 2) / 2);
        rt.proj.want(rt.f32_bytes((size_t)tiles_in_ * 16));
        rt.cat.want(rt.act_bytes(o_pad_));
        sh_->queries.want(rt.act_bytes((size_t)a.heads * 2 * round_up(a.dim, 32)));
        rt.want_planes(o_pad_ / 32, true);
    }
    bool portion_cost(uint32_t n, uint32_t len, double& as_tokens, double& as_long) const override {
        if (!rt_.bf16() || most_queries_ < 64) return false;
        const double work = 2.0 * n * (len + n / 2.0) * a_.heads * 2 * (a_.dim + a_.vdim);
        as_tokens += 4.0 * work;              // pages come from memory once for 16 queries instead of 64 or 128
        as_long += work;
        return true;
    }
    uint32_t enqueue(const Rows& r) override {
        const uint32_t ld = tiles_in_ * 16;
        {
            M40llmPackedGemm g = rt_.product(rt_.h.ptr(), rt_.d_pad, w_in_, tiles_in_, rt_.d_pad / 32, r.rows, M40LLM_PACKED_STORE);
            g.out_f32 = rt_.proj.ptr(); g.ld_out = ld; g.cols = ld;
            rt_.launch(g);
        }
        DeviceBuf& cache = source_ ? source_->cache_ : cache_;
        {
            M40llmPairSplit s{};
            s.act_dtype = rt_.opt.act_dtype; s.rows = r.rows; s.maps = 2; s.heads = a_.heads; s.kv_heads = a_.kv_heads; s.dim = a_.dim; s.vdim = a_.vdim; s.taps = a_.taps;
            s.eps = rt_.spec.eps;
            s.proj = rt_.proj.ptr(); s.ld_proj = ld; s.k_offset = k_offset_; s.v_offset = v_offset_;
            s.q_conv = q_conv_.ptr(); s.k_conv = k_conv_.ptr(); s.v_conv = v_conv_.ptr();
            s.q_norm = q_norm_.ptr(); s.k_norm = k_norm_.ptr();
            s.conv_state = conv_state_.ptr(); s.ld_state = conv_cols_;
            s.queries = sh_->queries.ptr();
            s.cache = source_ ? nullptr : cache.ptr();
            s.row_slot = r.slot; s.row_pos = r.pos; s.row_back = r.back; s.page_table = r.page_table; s.max_pages = rt_.max_pages;
            M40H_TRY(m40llm_ext_pair_split_append_async(rt_.ctx, &s, rt_.kStream));
        }
        if (a_.taps > 1 && r.multi_row_portions)
            M40H_TRY(m40llm_ext_conv_state_async(rt_.ctx, rt_.proj.ptr(), ld, conv_cols_, a_.taps, conv_state_.ptr(), conv_cols_, portions_.multi(),
                                                 r.pos, r.multi_row_portions, rt_.kStream));
        M40llmPairAttention h{};
        h.act_dtype = rt_.opt.act_dtype; h.maps = 2; h.heads = a_.heads; h.kv_heads = a_.kv_heads; h.dim = a_.dim; h.vdim = a_.vdim;
        h.scale = std::fabs(a_.scale); h.lambda = lambda_; h.out_scale = (float)(1.0 - a_.diff); h.eps = rt_.spec.eps;
        h.queries = sh_->queries.ptr(); h.cache = cache.ptr();
        h.gate = rt_.proj.f32(gate_offset_); h.ld_gate = ld;
        h.row_slot = r.slot; h.row_pos = r.pos; h.page_table = r.page_table; h.max_pages = rt_.max_pages;
        h.out = rt_.cat.ptr(); h.ld_out = o_pad_;
        h.tile_queries = tiles_->long_queries; h.splits = 1; h.n_rows = r.rows;
        if (!rt_.bf16()) {
            M40H_TRY(m40llm_ext_pair_attention_async(rt_.ctx, &h, rt_.kStream));
        } else {
            if (tiles_->n_short) {
                M40llmPairAttention s = h;
                s.tiles = tiles_->at; s.n_tiles = tiles_->n_short; s.splits = tiles_->splits; s.n_rows = r.short_rows;
                s.partial = rt_.partial.ptr(); s.partial_floats = rt_.partial.bytes() / 4;
                M40H_TRY(m40llm_ext_pair_attention_async(rt_.ctx, &s, rt_.kStream));
            }
            if (tiles_->n_long) {
                h.form = 1;
                h.tiles = tiles_->long_tiles(); h.n_tiles = tiles_->n_long;
                M40H_TRY(m40llm_ext_pair_attention_async(rt_.ctx, &h, rt_.kStream));
            }
        }
        return rt_.into_planes(rt_.product(rt_.cat.ptr(), o_pad_, w_out_, round_up(rt_.spec.width, 16) / 16, o_pad_ / 32, r.rows, M40LLM_PACKED_STORE), r.rows);
    }

private:
    LayerRuntime& rt_;
    std::shared_ptr<PairShared> sh_;
    DifferentialAttentionSpec a_;
    DifferentialMixer* source_;           // whose cache it reads (null = its own)
    PortionTable& portions_;
    PairTiles* tiles_;
    uint32_t most_queries_, k_offset_, v_offset_, gate_offset_, conv_cols_, tiles_in_, o_pad_;
    float lambda_;
    DeviceBuf w_in_, q_norm_, k_norm_, q_conv_, k_conv_, v_conv_, w_out_, cache_, conv_state_;
};

struct LightningShared { Scratch qkv, o; DeviceBuf states; };

// Launches: product (gate logits | silu of queries, keys, values) | recurrence (longer bf16 portions: states, outputs) | norm and gate | product
class LightningMixer : public Mixer {
public:
    LightningMixer(LayerRuntime& rt, std::shared_ptr<LightningShared> shared, TensorSource& t, uint32_t index, const LightningSpec& a)
        : rt_(rt), sh_(std::move(shared)), a_(a), portions_(rt.portions()) {
        if (!m40llm_ext_lightning_serves(a.dim, a.vdim))
            throw std::invalid_argument("layer " + std::to_string(index) + ": head sizes beyond what the recurrence's kernels serve");
        const std::string p = "l" + std::to_string(index) + ".mix.";
        const uint32_t D = rt.spec.width, d_tiles = rt.d_pad / 32, dp = round_up(a.dim, 32), vp = round_up(a.vdim, 32);
        cols_ = a.heads * a.vdim;
        gate_tiles_ = round_up(cols_, 16) / 16;
        qkv_cols_ = a.heads * (2 * dp + vp);
        o_pad_ = round_up(cols_, 32);
        w_in_ = rt.packed(gate_tiles_ + qkv_cols_ / 16, d_tiles);
        rt.pack(t, p + "g", cols_, D, w_in_.ptr(), d_tiles, 0);
        uint32_t tile = gate_tiles_;
        for (const char* name : {"q", "k", "v"}) {
            const bool value = *name == 'v';
            const uint32_t n = value ? a.vdim : a.dim, pad = value ? vp : dp;
            rt.pack_heads(rt.stage(t, p + name, {(uint64_t)a.heads * n, D}), a.heads, n, 0, n, D, w_in_.ptr(), d_tiles, pad, 0, tile);
            tile += a.heads * pad / 16;
        }
        norm_ = rt.upload_f32(t.read_f32(p + "norm", {cols_}));
        w_out_ = rt.packed(round_up(D, 16) / 16, o_pad_ / 32);
        rt.pack(t, p + "o", D, cols_, w_out_.ptr(), o_pad_ / 32, 0);
        std::vector<float> decay, log2_decay;
        for (double d : a.decay) {
            decay.push_back((float)d);
            log2_decay.push_back((float)std::log2(d));
        }
        decay_ = rt.upload_f32(decay);
        log2_decay_ = rt.upload_f32(log2_decay);
        const size_t slot = (size_t)a.heads * a.dim * vp * 4;
        state_ = rt.cleared(slot * rt.opt.max_sequences);
        rt.states.push_back({&state_, slot});
        rt.proj.want(rt.f32_bytes((size_t)gate_tiles_ * 16));
        rt.cat.want(rt.act_bytes(o_pad_));
        sh_->qkv.want(rt.act_bytes(qkv_cols_));
        sh_->o.want(rt.f32_bytes(cols_));
        rt.want_planes(o_pad_ / 32, true);
    }
    void prepare(const Rows&) override {
        if (!rt_.bf16()) return;
        const uint64_t need = m40llm_ext_lightning_scratch_bytes(portions_.n_chunks, a_.heads, a_.dim, a_.vdim);
        if (need > sh_->states.bytes()) {
            M40H_TRY(m40llm_stream_synchronize(rt_.ctx, rt_.kStream));
            sh_->states = DeviceBuf(rt_.ctx, need);
        }
    }
    uint32_t enqueue(const Rows& r) override {
        const uint32_t ld = gate_tiles_ * 16;
        {
            M40llmPackedGemm g = rt_.product(rt_.h.ptr(), rt_.d_pad, w_in_, gate_tiles_ + qkv_cols_ / 16, rt_.d_pad / 32, r.rows, M40LLM_PACKED_SILU);
            g.plain_tiles = gate_tiles_;
            g.out_f32 = rt_.proj.ptr(); g.ld_out = ld;
            g.out_act = sh_->qkv.ptr(); g.ld_act = qkv_cols_;
            rt_.launch(g);
        }
        M40llmLightning l{};
        l.act_dtype = rt_.opt.act_dtype; l.heads = a_.heads; l.dim = a_.dim; l.vdim = a_.vdim;
        l.qkv = sh_->qkv.ptr(); l.ld_qkv = qkv_cols_;
        l.decay = decay_.ptr(); l.log2_decay = log2_decay_.ptr();
        l.state = state_.ptr(); l.o = sh_->o.ptr(); l.ld_o = cols_;
        l.row_pos = r.pos;
        if (portions_.singles) {
            l.portions = portions_.at; l.n_portions = portions_.singles;
            M40H_TRY(m40llm_ext_lightning_async(rt_.ctx, &l, rt_.kStream));
        }
        if (r.multi_row_portions) {
            l.chunked = rt_.bf16();
            l.portions = portions_.multi(); l.n_portions = r.multi_row_portions;
            l.chunk_base = portions_.chunk_base(); l.chunks = portions_.chunks(); l.n_chunks = portions_.n_chunks;
            l.scratch = sh_->states.ptr(); l.scratch_bytes = sh_->states.bytes();
            M40H_TRY(m40llm_ext_lightning_async(rt_.ctx, &l, rt_.kStream));
        }
        M40H_TRY(m40llm_ext_norm_gate_rows_async(rt_.ctx, sh_->o.ptr(), cols_, norm_.ptr(), rt_.proj.ptr(), ld, r.rows, cols_, rt_.spec.eps, rt_.cat.ptr(), o_pad_,
                                                 rt_.opt.act_dtype, rt_.kStream));
        return rt_.into_planes(rt_.product(rt_.cat.ptr(), o_pad_, w_out_, round_up(rt_.spec.width, 16) / 16, o_pad_ / 32, r.rows, M40LLM_PACKED_STORE), r.rows);
    }

private:
    LayerRuntime& rt_;
    std::shared_ptr<LightningShared> sh_;
    LightningSpec a_;
    PortionTable& portions_;
    uint32_t cols_, gate_tiles_, qkv_cols_, o_pad_;
    DeviceBuf w_in_, norm_, w_out_, decay_, log2_decay_, state_;
};

// Where a sublayer leaves its output for the launch that takes it to the residual: in planes, or as the experts' rows.
struct SublayerOut {
    const void* planes = nullptr;
    uint32_t n_planes = 0, top = 0;
    uint64_t plane_stride = 0;
    const void* expert_out = nullptr;
    uint64_t ld_expert = 0;
    const uint32_t* place = nullptr;
    const void* weight = nullptr;
    template <class N>
    void put(N& n) const {
        n.planes = planes; n.n_planes = n_planes; n.plane_stride = plane_stride;
        n.expert_out = expert_out; n.ld_expert = ld_expert; n.place = place; n.weight = weight; n.top = top;
    }
};

class FeedForward {
public:
    virtual ~FeedForward() = default;
    virtual SublayerOut enqueue(const Rows& r) = 0;
    virtual bool reads_plain_rows() const { return false; }      // it wants its input as plain rows (h_rows) as well
};

inline uint32_t activation_code(Activation a) { return a == Activation::LimitedGate ? M40LLM_LIMITED_GATE : a == Activation::Silu ? M40LLM_SILU : M40LLM_GELU_TANH; }

class DenseFeedForward : public FeedForward {
public:
    DenseFeedForward(LayerRuntime& rt, TensorSource& t, const std::string& layer, const GatedMlpSpec& m) : rt_(rt), m_(m) {
        const std::string p = layer + "mlp.";
        const uint32_t D = rt.spec.width, d_tiles = rt.d_pad / 32;
        tiles_ = round_up(m.ff, 16) / 16;
        pad_ = round_up(m.ff, 32);
        w_in_ = rt.packed(2 * tiles_, d_tiles);
        rt.pack(t, p + "gate", m.ff, D, w_in_.ptr(), d_tiles, 0, 0, 2);
        rt.pack(t, p + "up", m.ff, D, w_in_.ptr(), d_tiles, 1, 0, 2);
        w_out_ = rt.packed(round_up(D, 16) / 16, pad_ / 32);
        rt.pack(t, p + "down", D, m.ff, w_out_.ptr(), pad_ / 32, 0);
        rt.cat.want(rt.act_bytes(pad_));
        rt.want_planes(pad_ / 32, true);
    }
    SublayerOut enqueue(const Rows& r) override {
        SublayerOut n;
        M40llmPackedGemm g = rt_.product(rt_.h.ptr(), rt_.d_pad, w_in_, 2 * tiles_, rt_.d_pad / 32, r.rows, M40LLM_PACKED_PROJECT);
        g.activation = activation_code(m_.activation);
        g.out_act = rt_.cat.ptr(); g.ld_act = pad_;
        rt_.launch(g);
        n.planes = rt_.planes.ptr();
        n.n_planes = rt_.into_planes(rt_.product(rt_.cat.ptr(), pad_, w_out_, round_up(rt_.spec.width, 16) / 16, pad_ / 32, r.rows, M40LLM_PACKED_STORE), r.rows);
        n.plane_stride = (uint64_t)r.rows * rt_.spec.width;
        return n;
    }

private:
    LayerRuntime& rt_;
    GatedMlpSpec m_;
    uint32_t tiles_, pad_;
    DeviceBuf w_in_, w_out_;
};

// Launches: product | polynomial | product
class PolyFeedForward : public FeedForward {
public:
    PolyFeedForward(LayerRuntime& rt, TensorSource& t, const std::string& layer, const PolyMlpSpec& m) : rt_(rt), m_(m), pad_(round_up(m.ff, 32)) {
        const std::string p = layer + "mlp.";
        const uint32_t D = rt.spec.width, d_tiles = rt.d_pad / 32;
        w_in_ = rt.packed(pad_ / 16, d_tiles);             // columns past ff are zeros, which the norms' sums need
        rt.pack(t, p + "up", m.ff, D, w_in_.ptr(), d_tiles, 0);
        act_ = rt.upload_f32(t.read_f32(p + "act", {4}));
        w_out_ = rt.packed(round_up(D, 16) / 16, pad_ / 32);
        rt.pack(t, p + "down", D, m.ff, w_out_.ptr(), pad_ / 32, 0);
        rt.cat.want(rt.act_bytes(pad_));
        rt.want_planes(pad_ / 32, true);
    }
    SublayerOut enqueue(const Rows& r) override {
        SublayerOut n;
        M40llmPackedGemm g = rt_.product(rt_.h.ptr(), rt_.d_pad, w_in_, pad_ / 16, rt_.d_pad / 32, r.rows, M40LLM_PACKED_SPLIT);
        g.out_act = rt_.cat.ptr(); g.ld_act = pad_;
        rt_.launch(g);
        M40H_TRY(m40llm_ext_poly_norm_rows_async(rt_.ctx, rt_.cat.ptr(), pad_, act_.ptr(), r.rows, m_.ff, rt_.spec.eps, rt_.opt.act_dtype, rt_.kStream));
        n.planes = rt_.planes.ptr();
        n.n_planes = rt_.into_planes(rt_.product(rt_.cat.ptr(), pad_, w_out_, round_up(rt_.spec.width, 16) / 16, pad_ / 32, r.rows, M40LLM_PACKED_STORE), r.rows);
        n.plane_stride = (uint64_t)r.rows * rt_.spec.width;
        return n;
    }

private:
    LayerRuntime& rt_;
    PolyMlpSpec m_;
    uint32_t pad_;
    DeviceBuf w_in_, act_, w_out_;
};

struct ExpertShared { Scratch logits, ids, weight, rows_of, place, jobs, rows, act, out, slot_weight; };

// Launches: product (router logits) | choice and sorted list (two launches above 64 rows) | (many rows: rows in list order) | gate and up per
// expert | down per expert
class ExpertFeedForward : public FeedForward {
public:
    ExpertFeedForward(LayerRuntime& rt, std::shared_ptr<ExpertShared> shared, TensorSource& t, const std::string& layer, const ExpertMlpSpec& m)
        : rt_(rt), sh_(std::move(shared)), m_(m) {
        const std::string p = layer + "mlp.", where = "layer " + layer.substr(1, layer.size() - 2) + ": ";
        const uint32_t D = rt.spec.width, d_tiles = rt.d_pad / 32, all = m.experts + m.identity;
        if (all > M40LLM_MAX_EXPERTS) throw std::invalid_argument(where + "more experts than the routing kernels serve");
        tiles_ = round_up(m.ff, 16) / 16;
        pad_ = round_up(m.ff, 32);
        out_cols_ = round_up(D, 8);
        router_tiles_ = round_up(all, 16) / 16;
        w_router_ = rt.packed(router_tiles_, d_tiles);
        rt.pack(t, p + "router", all, D, w_router_.ptr(), d_tiles, 0);
        if (m.correction) correction_ = rt.upload_f32(t.read_f32(p + "correction", {all}));
        const uint32_t down_tiles = round_up(D, 16) / 16;
        w_in_ = rt.packed(m.experts * 2 * tiles_, d_tiles);
        w_out_ = rt.packed(m.experts * down_tiles, pad_ / 32);
        for (uint32_t e = 0; e < m.experts; ++e) {
            const std::string pe = p + "e" + std::to_string(e) + ".";
            rt.pack(t, pe + "gate", m.ff, D, w_in_.ptr(), d_tiles, e * 2 * tiles_, 0, 2);
            rt.pack(t, pe + "up", m.ff, D, w_in_.ptr(), d_tiles, e * 2 * tiles_ + 1, 0, 2);
            rt.pack(t, pe + "down", D, m.ff, w_out_.ptr(), pad_ / 32, e * down_tiles);
        }
        const uint32_t R = rt.rows_pad, slots = m40llm_ext_expert_slots(R, m.experts, m.top);
        if (slots == 0 || m40llm_ext_expert_max_jobs(R, m.experts, m.top, 16) == 0) throw std::invalid_argument(where + "too many rows times experts a step");
        rt.h_rows.want(rt.act_bytes(rt.d_pad));
        sh_->logits.want(rt.f32_bytes((size_t)router_tiles_ * 16));
        sh_->ids.want((size_t)R * m.top * 4);
        sh_->weight.want((size_t)R * m.top * 4);
        sh_->place.want((size_t)R * m.top * 4);
        sh_->rows_of.want((size_t)slots * 4);
        sh_->jobs.want(16 + (size_t)m40llm_ext_expert_max_jobs(R, m.experts, m.top, 16) * 16);
        if (rt.bf16() && rows_a_job(R) == 128) sh_->rows.want((size_t)slots * rt.d_pad * rt.es);
        sh_->act.want((size_t)slots * pad_ * rt.es);
        sh_->out.want((size_t)slots * out_cols_ * rt.es);
        if (m.weight_input) sh_->slot_weight.want((size_t)slots * 4);
    }
    bool reads_plain_rows() const override { return true; }
    SublayerOut enqueue(const Rows& r) override {
        SublayerOut n;
        {
            M40llmPackedGemm g = rt_.product(rt_.h.ptr(), rt_.d_pad, w_router_, router_tiles_, rt_.d_pad / 32, r.rows, M40LLM_PACKED_STORE);
            g.out_f32 = sh_->logits.ptr(); g.ld_out = router_tiles_ * 16; g.cols = router_tiles_ * 16;
            rt_.launch(g);
        }
        const uint32_t job_rows = rows_a_job(r.rows), max_jobs = m40llm_ext_expert_max_jobs(r.rows, m_.experts, m_.top, job_rows);
        {
            M40llmRoute q{};
            q.rows = r.rows; q.experts = m_.experts; q.identity = m_.identity; q.top = m_.top; q.job_rows = job_rows; q.groups = m_.groups; q.keep = m_.keep; q.scale = m_.scale;
            q.logits = sh_->logits.ptr(); q.ld_logits = router_tiles_ * 16; q.correction = correction_.ptr();
            q.ids = sh_->ids.u32(); q.weight = sh_->weight.ptr();
            q.rows_of = sh_->rows_of.u32(); q.place = sh_->place.u32(); q.jobs = sh_->jobs.u32();
            q.score = m_.score == RouterScore::Sigmoid ? M40LLM_SCORE_SIGMOID : M40LLM_SCORE_SOFTMAX;
            if (m_.weight_input) q.slot_weight = sh_->slot_weight.ptr();
            M40H_TRY(m40llm_ext_route_rows_async(rt_.ctx, &q, rt_.kStream));
        }
        const uint32_t d_tiles = rt_.d_pad / 32, down_tiles = round_up(rt_.spec.width, 16) / 16;
        {
            M40llmPackedGemm g = rt_.product(rt_.h_rows.ptr(), rt_.d_pad, w_in_, 2 * tiles_, d_tiles, r.rows, M40LLM_PACKED_PROJECT);
            g.activation = activation_code(m_.activation);
            g.act_limit = m_.limit; g.act_alpha = m_.alpha;
            if (m_.weight_input) g.row_scale = sh_->slot_weight.ptr();      // gate and up are linear in the input
            if (job_rows == 128) {
                M40H_TRY(m40llm_ext_gather_rows_async(rt_.ctx, rt_.h_rows.ptr(), rt_.d_pad, sh_->rows_of.u32(), sh_->jobs.u32(),
                                                      m40llm_ext_expert_slots(r.rows, m_.experts, m_.top), sh_->rows.ptr(), rt_.kStream));
                g.a = sh_->rows.ptr();
            } else {
                g.gather = sh_->rows_of.u32();
            }
            g.jobs = sh_->jobs.u32(); g.max_jobs = max_jobs; g.job_rows = job_rows;
            g.w_batch = (uint64_t)2 * tiles_ * d_tiles * 512;
            g.out_act = sh_->act.ptr(); g.ld_act = pad_;
            rt_.launch(g);
        }
        {
            M40llmPackedGemm g = rt_.product(sh_->act.ptr(), pad_, w_out_, down_tiles, pad_ / 32, r.rows, M40LLM_PACKED_STORE_ACT);
            g.jobs = sh_->jobs.u32(); g.max_jobs = max_jobs; g.job_rows = job_rows;
            g.w_batch = (uint64_t)down_tiles * (pad_ / 32) * 512;
            g.out_act = sh_->out.ptr(); g.ld_act = out_cols_; g.cols = rt_.spec.width;
            rt_.launch(g);
        }
        n.expert_out = sh_->out.ptr(); n.ld_expert = out_cols_;
        n.place = sh_->place.u32(); n.top = m_.top;
        n.weight = m_.weight_input ? nullptr : sh_->weight.ptr();
        return n;
    }

private:
    // by the rows an expert gets on average
    uint32_t rows_a_job(uint32_t rows) const {
        const uint32_t mean = (uint32_t)((uint64_t)rows * m_.top / m_.experts);
        if (rows <= 16 || mean <= 12) return 16;
        if (rt_.bf16() && rows > 64 && mean >= 48) return 128;
        return mean <= 24 ? 32 : 64;
    }
    LayerRuntime& rt_;
    std::shared_ptr<ExpertShared> sh_;
    ExpertMlpSpec m_;
    uint32_t tiles_, pad_, out_cols_, router_tiles_;
    DeviceBuf w_router_, correction_, w_in_, w_out_;
};

class OutputNormLayer : public DecoderLayer {
public:
    OutputNormLayer(LayerRuntime& rt, TensorSource& t, uint32_t index, std::unique_ptr<Mixer> mixer, std::unique_ptr<FeedForward> ff)
        : rt_(rt), mixer_(std::move(mixer)), ff_(std::move(ff)) {
        const std::string p = "l" + std::to_string(index) + ".";
        norm1_ = rt.upload_f32(t.read_f32(p + "norm1", {rt.spec.width}));
        if (ff_) norm2_ = rt.upload_f32(t.read_f32(p + "norm2", {rt.spec.width}));
    }
    void prepare(const Rows& r) override { mixer_->prepare(r); }
    bool portion_cost(uint32_t n, uint32_t len, double& as_tokens, double& as_long) const override { return mixer_->portion_cost(n, len, as_tokens, as_long); }
    void enqueue(const Rows& r) override {
        M40llmNormAdd n{};
        n.act_dtype = rt_.opt.act_dtype; n.rows = r.rows; n.width = rt_.spec.width;
        n.eps = rt_.spec.eps; n.mult = rt_.spec.residual_mult;
        n.x = rt_.x.ptr();
        n.h = rt_.h.ptr(); n.ld_h = rt_.d_pad;
        M40llmNormAdd m = n;
        m.n_planes = mixer_->enqueue(r);
        m.planes = rt_.planes.ptr(); m.plane_stride = (uint64_t)r.rows * rt_.spec.width;
        m.w = norm1_.ptr();
        m.h_rows = ff_ && ff_->reads_plain_rows() ? rt_.h_rows.ptr() : nullptr;
        M40H_TRY(m40llm_ext_norm_add_rows_async(rt_.ctx, &m, rt_.kStream));
        if (!ff_) return;
        ff_->enqueue(r).put(n);
        n.w = norm2_.ptr();
        M40H_TRY(m40llm_ext_norm_add_rows_async(rt_.ctx, &n, rt_.kStream));
    }

private:
    LayerRuntime& rt_;
    std::unique_ptr<Mixer> mixer_;
    std::unique_ptr<FeedForward> ff_;
    DeviceBuf norm1_, norm2_;
};

}  // namespace m40host
