// Layers over residual streams: every sublayer reads a weighted sum of the streams behind a norm, and every stream takes a mixture of all old
// ones and its share of the output; a pre-norm layer is one over a single stream that takes all of it.  Mixers: softmax attention, attention beside a
// matrix memory, a delta rule, time mixing, a state space layer.
#pragma once

#include "output_norm_layer.hpp"

namespace m40host {

struct StreamWeights { DeviceBuf mix, share, take, norm; };       // of one sublayer

// The streams of a pass and what of the sublayer before they have not taken yet.
class ResidualStreams {
public:
    explicit ResidualStreams(LayerRuntime& rt) : rt_(rt), stride_((uint64_t)rt.rows_pad * rt.spec.width) {
        x_ = rt.cleared((size_t)stride_ * rt.spec.streams * 4);
    }
    StreamWeights load(TensorSource& t, const std::string& layer, const char* q) {
        const uint32_t s = rt_.spec.streams;
        const std::string p = layer + "hc" + q + ".";
        StreamWeights w;
        if (rt_.spec.block == BlockKind::PreNorm) {
            w.mix = rt_.upload_f32({1.0f}); w.share = rt_.upload_f32({1.0f}); w.take = rt_.upload_f32({1.0f});
            w.norm = rt_.upload_norm(t, layer + "norm" + q);
            return w;
        }
        w.mix = rt_.upload_f32(t.read_f32(p + "mix", {s, s}));
        w.share = rt_.upload_f32(t.read_f32(p + "out", {s}));
        w.take = rt_.upload_f32(t.read_f32(p + "in", {s}));
        w.norm = rt_.upload_norm(t, layer + "norm" + q);
        return w;
    }
    void begin() { fresh_ = true; pending_ = nullptr; }          // all streams are the embedding's rows
    // what the sublayer of these weights reads, as packed (and plain) rows
    void read(const Rows& r, const StreamWeights& w, bool plain_rows) {
        M40llmStreamUpdate u = update(r.rows);
        u.take = w.take.ptr(); u.w = w.norm.ptr();
        u.h = rt_.h.ptr(); u.ld_h = rt_.d_pad;
        u.h_rows = plain_rows ? rt_.h_rows.ptr() : nullptr;
        M40H_TRY(m40llm_ext_stream_update_async(rt_.ctx, &u, rt_.kStream));
        taken();
    }
    void write(const StreamWeights& w, const SublayerOut& out) { pending_ = &w; out_ = out; }
    // the streams' sum to x: of all rows, the streams kept ...
    void sum(const Rows& r) {
        M40llmStreamUpdate u = update(r.rows);
        u.x_out = rt_.x.ptr();
        M40H_TRY(m40llm_ext_stream_update_async(rt_.ctx, &u, rt_.kStream));
        taken();
    }
    // ... or at the end, of n rows (row_index NULL = the first n), nothing kept
    void last_sum(const uint32_t* row_index, uint32_t n) {
        M40llmStreamUpdate u = update(n);
        u.x_out = rt_.x.ptr(); u.row_index = row_index; u.discard = 1;
        M40H_TRY(m40llm_ext_stream_update_async(rt_.ctx, &u, rt_.kStream));
    }

private:
    M40llmStreamUpdate update(uint32_t rows) const {
        M40llmStreamUpdate u{};
        u.act_dtype = rt_.opt.act_dtype; u.rows = rows; u.width = rt_.spec.width; u.streams = rt_.spec.streams;
        u.eps = rt_.spec.eps; u.mult = rt_.spec.residual_mult;
        u.x0 = fresh_ ? rt_.x.ptr() : nullptr;
        u.streams_x = x_.ptr(); u.stream_stride = stride_;
        if (pending_) {
            u.mix = pending_->mix.ptr(); u.share = pending_->share.ptr();
            out_.put(u);
        }
        return u;
    }
    void taken() {
        if (pending_) fresh_ = false;
        pending_ = nullptr;
    }
    LayerRuntime& rt_;
    uint64_t stride_;
    DeviceBuf x_;
    bool fresh_ = true;
    const StreamWeights* pending_ = nullptr;
    SublayerOut out_;
};

struct StreamShared {         // buffers the layers of a decoder share
    Scratch queries, first_values, recurrent, low, low_act, mixes, heads;
    DeviceBuf chunks;
};

// Softmax attention as part of a mixer: columns [queries | keys | values | gate] of its projections, from column 0 of proj on, and its heads from
// column 0 of the mixer's output operand on.
class AttentionPart {
public:
    // row tiles of the input product that are its own
    static uint32_t input_tiles(const AttentionSpec& a) { return gate_offset(a) / 16 + (a.column_gate ? round_up(a.heads * a.vdim, 16) / 16 : 0); }

    // twin: a part with the same tensors
    AttentionPart(LayerRuntime& rt, StreamShared& sh, TensorSource& t, const std::string& where, const std::string& p, const AttentionSpec& a, float out_factor,
                  bool takes_first_values, const AttentionPart* twin = nullptr)
        : rt_(rt), sh_(sh), a_(a), out_factor_(out_factor), takes_first_(takes_first_values), w_(twin ? twin->w_ : load(rt, t, p, a)) {
        most_queries_ = m40llm_ext_pair_attention_tile_queries(rt.opt.act_dtype, 1, a.dim, a.vdim);
        if (most_queries_ == 0) throw std::invalid_argument(where + "head sizes beyond what the attention kernels serve");
        if (a.rotation) rot_ = &rt.table<RotationAngles>(&rt, *a.rotation, std::max(a.rotation->dims / 2, 1u));
        if (takes_first_) lambda_ = t.read_f32(p + "vmix", {})[0];
        cache_ = rt.cleared((size_t)rt.max_pages * m40llm_ext_pair_page_elements(1, a.kv_heads, a.dim, a.vdim) * rt.es);
        tiles_ = &rt.table<PairTiles>(a.heads / a.kv_heads, most_queries_, a.window);
        tiles_->fewest_kv_heads = std::min(tiles_->fewest_kv_heads, a.kv_heads);
        tiles_->floats_a_row = std::max(tiles_->floats_a_row, m40llm_ext_pair_attention_partial_floats(1, 1, a.heads, a.vdim, 2) / 2);
        sh_.queries.want(rt.act_bytes((size_t)a.heads * round_up(a.dim, 32)));
        if (a.share_values) sh_.first_values.want(rt.f32_bytes(a.kv_heads * a.vdim));
    }
    void pack(TensorSource& t, const std::string& p, const DeviceBuf& w, uint32_t d_tiles) {
        const uint32_t D = rt_.spec.width;
        rt_.pack(t, p + "q", a_.heads * a_.dim, D, w.ptr(), d_tiles, 0);
        rt_.pack(t, p + "k", a_.kv_heads * a_.dim, D, w.ptr(), d_tiles, k_offset(a_) / 16);
        rt_.pack(t, p + "v", a_.kv_heads * a_.vdim, D, w.ptr(), d_tiles, v_offset(a_) / 16);
        if (a_.column_gate) rt_.pack(t, p + "g", a_.heads * a_.vdim, D, w.ptr(), d_tiles, gate_offset(a_) / 16);
    }
    bool portion_cost(uint32_t n, uint32_t len, double& as_tokens, double& as_long) const {
        if (!rt_.bf16() || most_queries_ < 64) return false;
        const double keys = len + n / 2.0, work = 2.0 * n * (a_.window ? std::min(keys, (double)a_.window) : keys) * a_.heads * (a_.dim + a_.vdim);
        as_tokens += 4.0 * work;              // pages come from memory once for 16 queries instead of 64 or 128
        as_long += work;
        return true;
    }
    void enqueue(const Rows& r, uint32_t ld, uint32_t ld_out) {
        if (a_.head_norm) {
            M40llmPairSplit s{};
            s.act_dtype = rt_.opt.act_dtype; s.rows = r.rows; s.maps = 1; s.heads = a_.heads; s.kv_heads = a_.kv_heads; s.dim = a_.dim; s.vdim = a_.vdim;
            s.eps = rt_.spec.eps;
            s.proj = rt_.proj.ptr(); s.ld_proj = ld; s.k_offset = k_offset(a_); s.v_offset = v_offset(a_);
            s.q_norm = w_->q_norm.ptr(); s.k_norm = w_->k_norm.ptr();
            s.queries = sh_.queries.ptr(); s.cache = cache_.ptr();
            s.row_slot = r.slot; s.row_pos = r.pos; s.row_back = r.back; s.page_table = r.page_table; s.max_pages = rt_.max_pages;
            M40H_TRY(m40llm_ext_pair_split_append_async(rt_.ctx, &s, rt_.kStream));
        } else {
            M40llmQkvSplit s{};
            s.act_dtype = rt_.opt.act_dtype; s.rows = r.rows; s.heads = a_.heads; s.kv_heads = a_.kv_heads; s.dim = a_.dim; s.vdim = a_.vdim;
            s.eps = rt_.spec.eps; s.q_factor = a_.scale < 0.0f ? -1.0f : 1.0f;        // the kernels take the scale's sign from the queries
            s.proj = rt_.proj.ptr(); s.ld_proj = ld; s.k_offset = k_offset(a_); s.v_offset = v_offset(a_);
            s.q_bias = w_->q_bias.ptr(); s.k_bias = w_->k_bias.ptr(); s.v_bias = w_->v_bias.ptr();
            s.q_norm = w_->q_norm.ptr(); s.k_norm = w_->k_norm.ptr();
            if (rot_) { s.angles = rot_->angles.ptr(); s.rot_half = rot_->half; }
            if (a_.share_values) {
                s.ld_values = a_.kv_heads * a_.vdim;
                if (takes_first_) { s.first_values = sh_.first_values.ptr(); s.lambda = lambda_; }
                else s.keep_values = sh_.first_values.ptr();
            }
            s.queries = sh_.queries.ptr(); s.cache = cache_.ptr();
            s.row_slot = r.slot; s.row_pos = r.pos; s.page_table = r.page_table; s.max_pages = rt_.max_pages;
            M40H_TRY(m40llm_ext_qkv_split_append_async(rt_.ctx, &s, rt_.kStream));
        }
        M40llmPairAttention h{};
        h.act_dtype = rt_.opt.act_dtype; h.maps = 1; h.heads = a_.heads; h.kv_heads = a_.kv_heads; h.dim = a_.dim; h.vdim = a_.vdim;
        h.scale = std::fabs(a_.scale); h.out_scale = out_factor_;
        h.window = a_.window; h.cap = a_.cap; h.slopes = w_->slopes.ptr(); h.sink = w_->sink.ptr();
        if (a_.head_norm) h.most = 1.02f * (float)a_.dim;        // both of length sqrt(dim) at most, then rounded
        h.queries = sh_.queries.ptr(); h.cache = cache_.ptr();
        if (a_.column_gate) { h.gate = rt_.proj.f32(gate_offset(a_)); h.ld_gate = ld; }
        h.row_slot = r.slot; h.row_pos = r.pos; h.page_table = r.page_table; h.max_pages = rt_.max_pages;
        h.out = rt_.cat.ptr(); h.ld_out = ld_out;
        h.tile_queries = tiles_->long_queries; h.splits = 1; h.n_rows = r.rows;
        if (!rt_.bf16()) {
            M40H_TRY(m40llm_ext_pair_attention_async(rt_.ctx, &h, rt_.kStream));
            return;
        }
        if (tiles_->n_short) {
            M40llmPairAttention s = h;
            s.tiles = tiles_->at; s.n_tiles = tiles_->n_short; s.splits = tiles_->splits; s.n_rows = r.short_rows;
            s.partial = rt_.partial.ptr(); s.partial_floats = rt_.partial.bytes() / 4;
            M40H_TRY(m40llm_ext_pair_attention_async(rt_.ctx, &s, rt_.kStream));
        }
        if (tiles_->n_long) {
            h.form = 1;
            h.tiles = tiles_->long_tiles(); h.n_tiles = tiles_->n_long; h.even = tiles_->even;
            M40H_TRY(m40llm_ext_pair_attention_async(rt_.ctx, &h, rt_.kStream));
        }
    }

private:
    struct Weights { DeviceBuf q_bias, k_bias, v_bias, q_norm, k_norm, slopes, sink; };
    static std::shared_ptr<const Weights> load(LayerRuntime& rt, TensorSource& t, const std::string& p, const AttentionSpec& a) {
        const uint32_t q = a.heads * a.dim, k = a.kv_heads * a.dim, v = a.kv_heads * a.vdim;
        auto w = std::make_shared<Weights>();
        if (a.biases) {
            w->q_bias = rt.upload_f32(t.read_f32(p + "q.b", {q}));
            w->k_bias = rt.upload_f32(t.read_f32(p + "k.b", {k}));
            w->v_bias = rt.upload_f32(t.read_f32(p + "v.b", {v}));
        }
        if (a.projection_norm) {
            w->q_norm = rt.upload_f32(t.read_f32(p + "q.norm", {q}));
            w->k_norm = rt.upload_f32(t.read_f32(p + "k.norm", {k}));
        }
        if (a.head_norm) {               // no weights; the kernels take the scale's sign from the queries
            w->q_norm = rt.upload_f32(std::vector<float>(a.dim, a.scale < 0.0f ? -1.0f : 1.0f));
            w->k_norm = rt.upload_f32(std::vector<float>(a.dim, 1.0f));
        }
        if (a.distance_slopes) {
            std::vector<float> s(a.heads);
            for (uint32_t h = 0; h < a.heads; ++h) s[h] = (float)std::exp2(-8.0 * (h + 1) / a.heads);
            w->slopes = rt.upload_f32(s);
        }
        if (a.sink) w->sink = rt.upload_f32(t.read_f32(p + "sink", {a.heads}));
        return w;
    }
    static uint32_t k_offset(const AttentionSpec& a) { return round_up(a.heads * a.dim, 16); }
    static uint32_t v_offset(const AttentionSpec& a) { return k_offset(a) + round_up(a.kv_heads * a.dim, 16); }
    static uint32_t gate_offset(const AttentionSpec& a) { return v_offset(a) + round_up(a.kv_heads * a.vdim, 16); }
    LayerRuntime& rt_;
    StreamShared& sh_;
    AttentionSpec a_;
    float out_factor_, lambda_ = 0.0f;
    bool takes_first_;
    std::shared_ptr<const Weights> w_;
    RotationAngles* rot_ = nullptr;
    PairTiles* tiles_;
    uint32_t most_queries_;
    DeviceBuf cache_;
};

// What recurrences do with a step's portions: single rows token after token, longer ones of bf16 passes chunk by chunk.
class RecurrentRows {
public:
    RecurrentRows(LayerRuntime& rt, StreamShared& sh) : rt_(rt), sh_(sh), portions_(rt.portions()) {}
    void prepare(uint32_t rule, uint32_t heads, uint32_t dim, uint32_t vdim) { prepare(m40llm_ext_memory_scratch_bytes(rule, portions_.n_chunks, heads, dim, vdim)); }
    void prepare(uint64_t need) {
        if (!rt_.bf16() || portions_.n_chunks == 0) return;
        if (need > sh_.chunks.bytes()) {
            M40H_TRY(m40llm_stream_synchronize(rt_.ctx, rt_.kStream));
            sh_.chunks = DeviceBuf(rt_.ctx, need);
        }
    }
    template <class P>
    void enqueue(const Rows& r, P p, int (*launch)(M40llmCudaContext*, const P*, uint32_t)) {
        p.row_pos = r.pos;
        if (portions_.singles) {
            p.portions = portions_.at; p.n_portions = portions_.singles;
            M40H_TRY(launch(rt_.ctx, &p, rt_.kStream));
        }
        if (r.multi_row_portions) {
            p.chunked = rt_.bf16();
            p.portions = portions_.multi(); p.n_portions = r.multi_row_portions;
            p.chunk_base = portions_.chunk_base(); p.chunks = portions_.chunks(); p.n_chunks = portions_.n_chunks;
            p.scratch = sh_.chunks.ptr(); p.scratch_bytes = sh_.chunks.bytes();
            M40H_TRY(launch(rt_.ctx, &p, rt_.kStream));
        }
    }
    const PortionTable& portions() const { return portions_; }
    const uint32_t* multi() const { return portions_.multi(); }

private:
    LayerRuntime& rt_;
    StreamShared& sh_;
    PortionTable& portions_;
};

// Launches: product (projections) | norms and cache append | attention | product
class AttentionMixer : public Mixer {
public:
    // twin: a mixer with the same tensors
    AttentionMixer(LayerRuntime& rt, std::shared_ptr<StreamShared> shared, TensorSource& t, uint32_t index, const AttentionSpec& a, bool takes_first_values,
                   const AttentionMixer* twin = nullptr)
        : rt_(rt), sh_(std::move(shared)), tiles_in_(AttentionPart::input_tiles(a)), o_pad_(round_up(a.heads * a.vdim, 32)) {
        const std::string where = "layer " + std::to_string(index) + ": ", p = "l" + std::to_string(index) + ".mix.";
        attention_ = std::make_unique<AttentionPart>(rt, *sh_, t, where, p, a, 1.0f, takes_first_values, twin ? twin->attention_.get() : nullptr);
        if (twin) {
            w_ = twin->w_;
        } else {
            w_ = std::make_shared<Weights>();
            w_->in = rt.packed(tiles_in_, rt.d_pad / 32);
            attention_->pack(t, p, w_->in, rt.d_pad / 32);
            w_->out = rt.packed(round_up(rt.spec.width, 16) / 16, o_pad_ / 32);
            rt.pack(t, p + "o", rt.spec.width, a.heads * a.vdim, w_->out.ptr(), o_pad_ / 32, 0);
        }
        rt.proj.want(rt.f32_bytes((size_t)tiles_in_ * 16));
        rt.cat.want(rt.act_bytes(o_pad_));
        rt.want_planes(o_pad_ / 32, true);
    }
    bool portion_cost(uint32_t n, uint32_t len, double& as_tokens, double& as_long) const override { return attention_->portion_cost(n, len, as_tokens, as_long); }
    uint32_t enqueue(const Rows& r) override {
        const uint32_t ld = tiles_in_ * 16;
        M40llmPackedGemm g = rt_.product(rt_.h.ptr(), rt_.d_pad, w_->in, tiles_in_, rt_.d_pad / 32, r.rows, M40LLM_PACKED_STORE);
        g.out_f32 = rt_.proj.ptr(); g.ld_out = ld; g.cols = ld;
        rt_.launch(g);
        attention_->enqueue(r, ld, o_pad_);
        return rt_.into_planes(rt_.product(rt_.cat.ptr(), o_pad_, w_->out, round_up(rt_.spec.width, 16) / 16, o_pad_ / 32, r.rows, M40LLM_PACKED_STORE), r.rows);
    }

private:
    struct Weights { DeviceBuf in, out; };
    LayerRuntime& rt_;
    std::shared_ptr<StreamShared> sh_;
    uint32_t tiles_in_, o_pad_;
    std::unique_ptr<AttentionPart> attention_;
    std::shared_ptr<Weights> w_;
};

// Launches: product (both sides' projections) | rotation and cache append | attention | matrix memory (norm and gate included) | product over both
// sides' heads, which carry their factors
class ParallelMixer : public Mixer {
public:
    ParallelMixer(LayerRuntime& rt, std::shared_ptr<StreamShared> shared, TensorSource& t, uint32_t index, const ParallelSpec& s)
        : rt_(rt), sh_(std::move(shared)), m_(s.right), right_scale_(s.right_scale), rows_(rt, *sh_) {
        const std::string where = "layer " + std::to_string(index) + ": ", p = "l" + std::to_string(index) + ".mix.", x = p + "right.";
        if (!m40llm_ext_memory_serves(m_.dim, m_.vdim)) throw std::invalid_argument(where + "head sizes beyond what the recurrence's kernels serve");
        const uint32_t D = rt.spec.width, d_tiles = rt.d_pad / 32, q = m_.heads * m_.dim, v = m_.heads * m_.vdim;
        attention_ = std::make_unique<AttentionPart>(rt, *sh_, t, where, p + "left.", s.left, s.left_scale, false);
        uint32_t at = AttentionPart::input_tiles(s.left) * 16;
        auto part = [&](uint32_t n) { const uint32_t c = at; at += round_up(n, 16); return c; };
        q_col_ = part(q); k_col_ = part(q); v_col_ = part(v); g_col_ = part(v); i_col_ = part(m_.heads); f_col_ = part(m_.heads);
        tiles_in_ = at / 16;
        w_in_ = rt.packed(tiles_in_, d_tiles);
        attention_->pack(t, p + "left.", w_in_, d_tiles);
        const std::pair<const char*, std::pair<uint32_t, uint32_t>> parts[] = {{"q", {q, q_col_}}, {"k", {q, k_col_}}, {"v", {v, v_col_}}, {"g", {v, g_col_}},
                                                                               {"i", {m_.heads, i_col_}}, {"f", {m_.heads, f_col_}}};
        for (const auto& c : parts) rt.pack(t, x + c.first, c.second.first, D, w_in_.ptr(), d_tiles, c.second.second / 16);
        i_bias_ = rt.upload_f32(t.read_f32(x + "i.b", {m_.heads}));
        f_bias_ = rt.upload_f32(t.read_f32(x + "f.b", {m_.heads}));
        norm_ = rt.upload_f32(t.read_f32(x + "norm", {v}));
        left_pad_ = round_up(s.left.heads * s.left.vdim, 32);
        o_pad_ = left_pad_ + round_up(v, 32);
        w_out_ = rt.packed(round_up(D, 16) / 16, o_pad_ / 32);
        rt.pack(t, p + "left.o", D, s.left.heads * s.left.vdim, w_out_.ptr(), o_pad_ / 32, 0);
        rt.pack(t, x + "o", D, v, w_out_.ptr(), o_pad_ / 32, 0, left_pad_);
        const size_t slot = m40llm_ext_matrix_memory_state_floats(m_.dim, m_.vdim) * m_.heads * 4;
        state_ = rt.cleared(slot * rt.opt.max_sequences);
        rt.states.push_back({&state_, slot});
        rt.proj.want(rt.f32_bytes((size_t)tiles_in_ * 16));
        rt.cat.want(rt.act_bytes(o_pad_));
        rt.want_planes(o_pad_ / 32, true);
    }
    void prepare(const Rows&) override { rows_.prepare(M40LLM_RULE_MEMORY, m_.heads, m_.dim, m_.vdim); }
    bool portion_cost(uint32_t n, uint32_t len, double& as_tokens, double& as_long) const override { return attention_->portion_cost(n, len, as_tokens, as_long); }
    uint32_t enqueue(const Rows& r) override {
        const uint32_t ld = tiles_in_ * 16;
        M40llmPackedGemm g = rt_.product(rt_.h.ptr(), rt_.d_pad, w_in_, tiles_in_, rt_.d_pad / 32, r.rows, M40LLM_PACKED_STORE);
        g.out_f32 = rt_.proj.ptr(); g.ld_out = ld; g.cols = ld;
        rt_.launch(g);
        attention_->enqueue(r, ld, o_pad_);
        M40llmMatrixMemory m{};
        m.act_dtype = rt_.opt.act_dtype; m.heads = m_.heads; m.dim = m_.dim; m.vdim = m_.vdim;
        m.cap = m_.gate_cap; m.q_factor = (float)(1.0 / std::sqrt((double)m_.dim)); m.eps = rt_.spec.eps; m.out_factor = right_scale_;
        m.proj = rt_.proj.ptr(); m.ld_proj = ld;
        m.q_col = q_col_; m.k_col = k_col_; m.v_col = v_col_; m.g_col = g_col_; m.i_col = i_col_; m.f_col = f_col_;
        m.i_bias = i_bias_.ptr(); m.f_bias = f_bias_.ptr(); m.norm = norm_.ptr();
        m.state = state_.ptr();
        m.out = rt_.cat.ptr(); m.ld_out = o_pad_; m.out_col = left_pad_;
        rows_.enqueue(r, m, m40llm_ext_matrix_memory_async);
        return rt_.into_planes(rt_.product(rt_.cat.ptr(), o_pad_, w_out_, round_up(rt_.spec.width, 16) / 16, o_pad_ / 32, r.rows, M40LLM_PACKED_STORE), r.rows);
    }

private:
    LayerRuntime& rt_;
    std::shared_ptr<StreamShared> sh_;
    MatrixMemorySpec m_;
    float right_scale_;
    RecurrentRows rows_;
    uint32_t q_col_, k_col_, v_col_, g_col_, i_col_, f_col_, tiles_in_, left_pad_, o_pad_;
    std::unique_ptr<AttentionPart> attention_;
    DeviceBuf w_in_, i_bias_, f_bias_, norm_, w_out_, state_;
};

// Launches: product (queries, keys, values, write strengths | inner sides of the low-rank products) | product (their outer sides) | convolution, unit
// vectors | (convolution state of longer portions) | delta rule (norm and gate included) | product
class ChannelDeltaMixer : public Mixer {
public:
    ChannelDeltaMixer(LayerRuntime& rt, std::shared_ptr<StreamShared> shared, TensorSource& t, uint32_t index, const ChannelDeltaSpec& a)
        : rt_(rt), sh_(std::move(shared)), a_(a), rows_(rt, *sh_) {
        const std::string where = "layer " + std::to_string(index) + ": ", p = "l" + std::to_string(index) + ".mix.";
        if (!m40llm_ext_memory_serves(a.dim, a.vdim)) throw std::invalid_argument(where + "head sizes beyond what the recurrence's kernels serve");
        const uint32_t D = rt.spec.width, d_tiles = rt.d_pad / 32, k = a.kv_heads * a.dim, v = a.heads * a.vdim, dims = a.heads * a.dim;
        const uint32_t a_rank = (uint32_t)t.rows_of(p + "a1", a.vdim), g_rank = (uint32_t)t.rows_of(p + "g1", a.vdim);
        conv_cols_ = 2 * k + v;
        beta_col_ = round_up(conv_cols_, 16);
        plain_tiles_ = (beta_col_ + round_up(a.heads, 16)) / 16;
        a_pad_ = round_up(a_rank, 32);
        low_pad_ = a_pad_ + round_up(g_rank, 32);
        tiles_in_ = plain_tiles_ + low_pad_ / 16;
        w_in_ = rt.packed(tiles_in_, d_tiles);
        auto rows_at = [&](const std::string& name, uint32_t n, uint32_t row) {
            rt.pack_heads(rt.stage(t, p + name, {n, D}), 1, n, 0, n, D, w_in_.ptr(), d_tiles, n, row);
        };
        rows_at("q", k, 0);
        rows_at("k", k, k);
        rows_at("v", v, 2 * k);
        rows_at("b", a.heads, beta_col_);
        rows_at("a1", a_rank, plain_tiles_ * 16);
        rows_at("g1", g_rank, plain_tiles_ * 16 + a_pad_);
        g_col_ = round_up(dims, 16);
        tiles_low_ = g_col_ / 16 + round_up(v, 16) / 16;
        w_low_ = rt.packed(tiles_low_, low_pad_ / 32);
        rt.pack(t, p + "a2", dims, a_rank, w_low_.ptr(), low_pad_ / 32, 0);
        rt.pack(t, p + "g2", v, g_rank, w_low_.ptr(), low_pad_ / 32, g_col_ / 16, a_pad_);
        q_conv_ = rt.upload_taps(t, p + "q.conv", k, a.taps);
        k_conv_ = rt.upload_taps(t, p + "k.conv", k, a.taps);
        v_conv_ = rt.upload_taps(t, p + "v.conv", v, a.taps);
        A_log_ = rt.upload_f32(t.read_f32(p + "A_log", {a.heads}));
        dt_bias_ = rt.upload_f32(t.read_f32(p + "dt_bias", {dims}));
        norm_ = rt.upload_f32(t.read_f32(p + "norm", {a.vdim}));
        o_pad_ = round_up(v, 32);
        w_out_ = rt.packed(round_up(D, 16) / 16, o_pad_ / 32);
        rt.pack(t, p + "o", D, v, w_out_.ptr(), o_pad_ / 32, 0);
        if (a.taps > 1) {
            const size_t slot = (size_t)(a.taps - 1) * round_up(conv_cols_, 4) * 4;
            conv_state_ = rt.cleared(slot * rt.opt.max_sequences);
            rt.states.push_back({&conv_state_, slot});
        }
        const size_t slot = m40llm_ext_channel_delta_state_floats(a.dim, a.vdim) * a.heads * 4;
        state_ = rt.cleared(slot * rt.opt.max_sequences);
        rt.states.push_back({&state_, slot});
        rt.proj.want(rt.f32_bytes((size_t)plain_tiles_ * 16));
        rt.cat.want(rt.act_bytes(o_pad_));
        sh_->recurrent.want(rt.f32_bytes(round_up(conv_cols_, 4)));
        sh_->low_act.want(rt.act_bytes(low_pad_));
        sh_->low.want(rt.f32_bytes((size_t)tiles_low_ * 16));
        rt.want_planes(o_pad_ / 32, true);
    }
    void prepare(const Rows&) override { rows_.prepare(M40LLM_RULE_DELTA, a_.heads, a_.dim, a_.vdim); }
    uint32_t enqueue(const Rows& r) override {
        const uint32_t ld = plain_tiles_ * 16, ld_low = tiles_low_ * 16, ld_conv = round_up(conv_cols_, 4);
        {
            M40llmPackedGemm g = rt_.product(rt_.h.ptr(), rt_.d_pad, w_in_, tiles_in_, rt_.d_pad / 32, r.rows, M40LLM_PACKED_SPLIT);
            g.plain_tiles = plain_tiles_;
            g.out_f32 = rt_.proj.ptr(); g.ld_out = ld;
            g.out_act = sh_->low_act.ptr(); g.ld_act = low_pad_;
            rt_.launch(g);
        }
        {
            M40llmPackedGemm g = rt_.product(sh_->low_act.ptr(), low_pad_, w_low_, tiles_low_, low_pad_ / 32, r.rows, M40LLM_PACKED_STORE);
            g.out_f32 = sh_->low.ptr(); g.ld_out = ld_low; g.cols = ld_low;
            rt_.launch(g);
        }
        {
            M40llmDeltaSplit s{};
            s.rows = r.rows; s.heads = a_.heads; s.kv_heads = a_.kv_heads; s.dim = a_.dim; s.vdim = a_.vdim; s.taps = a_.taps;
            s.q_factor = (float)(1.0 / std::sqrt((double)a_.dim));
            s.proj = rt_.proj.ptr(); s.ld_proj = ld;
            s.q_conv = q_conv_.ptr(); s.k_conv = k_conv_.ptr(); s.v_conv = v_conv_.ptr();
            s.conv_state = conv_state_.ptr(); s.ld_state = ld_conv;
            s.out = sh_->recurrent.ptr(); s.ld_out = ld_conv;
            s.row_slot = r.slot; s.row_pos = r.pos; s.row_back = r.back;
            M40H_TRY(m40llm_ext_delta_split_async(rt_.ctx, &s, rt_.kStream));
        }
        if (a_.taps > 1 && r.multi_row_portions)
            M40H_TRY(m40llm_ext_conv_state_async(rt_.ctx, rt_.proj.ptr(), ld, conv_cols_, a_.taps, conv_state_.ptr(), ld_conv, rows_.multi(), r.pos,
                                                 r.multi_row_portions, rt_.kStream));
        M40llmChannelDelta m{};
        m.act_dtype = rt_.opt.act_dtype; m.heads = a_.heads; m.kv_heads = a_.kv_heads; m.dim = a_.dim; m.vdim = a_.vdim;
        m.q_factor = 1.0f; m.eps = rt_.spec.eps; m.out_factor = 1.0f;
        m.qkv = sh_->recurrent.ptr(); m.ld_qkv = ld_conv;
        m.low = sh_->low.ptr(); m.ld_low = ld_low; m.a_col = 0; m.g_col = g_col_;
        m.beta = rt_.proj.f32(beta_col_); m.ld_beta = ld;
        m.A_log = A_log_.ptr(); m.dt_bias = dt_bias_.ptr(); m.norm = norm_.ptr();
        m.state = state_.ptr();
        m.out = rt_.cat.ptr(); m.ld_out = o_pad_;
        rows_.enqueue(r, m, m40llm_ext_channel_delta_async);
        return rt_.into_planes(rt_.product(rt_.cat.ptr(), o_pad_, w_out_, round_up(rt_.spec.width, 16) / 16, o_pad_ / 32, r.rows, M40LLM_PACKED_STORE), r.rows);
    }

private:
    LayerRuntime& rt_;
    std::shared_ptr<StreamShared> sh_;
    ChannelDeltaSpec a_;
    RecurrentRows rows_;
    uint32_t conv_cols_, beta_col_, plain_tiles_, a_pad_, low_pad_, tiles_in_, g_col_, tiles_low_, o_pad_;
    DeviceBuf w_in_, w_low_, q_conv_, k_conv_, v_conv_, A_log_, dt_bias_, norm_, w_out_, conv_state_, state_;
};

class StreamLayer : public DecoderLayer {
public:
    StreamLayer(LayerRuntime& rt, ResidualStreams& streams, TensorSource& t, uint32_t index, std::unique_ptr<Mixer> mixer, std::unique_ptr<FeedForward> ff)
        : rt_(rt), streams_(streams), mixer_(std::move(mixer)) {
        const std::string p = "l" + std::to_string(index) + ".";
        auto w = std::make_shared<Weights>();
        w->ff = std::move(ff);
        w->mix = streams.load(t, p, "1");
        if (w->ff) w->feed = streams.load(t, p, "2");
        w_ = std::move(w);
    }
    // with the tensors of another layer, whose mixer this one's shares them with
    StreamLayer(const StreamLayer& twin, std::unique_ptr<Mixer> mixer) : rt_(twin.rt_), streams_(twin.streams_), mixer_(std::move(mixer)), w_(twin.w_) {}
    const Mixer* mixer() const { return mixer_.get(); }
    void prepare(const Rows& r) override { mixer_->prepare(r); }
    bool portion_cost(uint32_t n, uint32_t len, double& as_tokens, double& as_long) const override { return mixer_->portion_cost(n, len, as_tokens, as_long); }
    void enqueue(const Rows& r) override {
        streams_.read(r, w_->mix, mixer_->reads_plain_rows());
        SublayerOut y;
        y.n_planes = mixer_->enqueue(r);
        y.planes = rt_.planes.ptr(); y.plane_stride = (uint64_t)r.rows * rt_.spec.width;
        streams_.write(w_->mix, y);
        if (w_->ff) {
            streams_.read(r, w_->feed, w_->ff->reads_plain_rows());
            streams_.write(w_->feed, w_->ff->enqueue(r));
        }
        if (r.in_place) streams_.sum(r);
    }

private:
    LayerRuntime& rt_;
    struct Weights {
        StreamWeights mix, feed;
        std::unique_ptr<FeedForward> ff;
    };
    ResidualStreams& streams_;
    std::unique_ptr<Mixer> mixer_;
    std::shared_ptr<const Weights> w_;
};

}  // namespace m40host
