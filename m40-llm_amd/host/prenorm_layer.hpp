// Mixers of pre-norm layers: time mixing and state space layers.  Layers with the same tensors share them (twin) and have a state of their own.
#pragma once

#include "stream_layer.hpp"

namespace m40host {

// Launches: token mixes (and the row kept for the next portion) | product (receptance, keys, values, gates | inner side of the decays) | product (outer
// side) | recurrence (norm and gate included) | product
class TimeMixingMixer : public Mixer {
public:
    TimeMixingMixer(LayerRuntime& rt, std::shared_ptr<StreamShared> shared, TensorSource& t, uint32_t index, const TimeMixingSpec& a, const TimeMixingMixer* twin)
        : rt_(rt), sh_(std::move(shared)), a_(a), rows_(rt, *sh_), w_(twin ? twin->w_ : load(rt, t, "l" + std::to_string(index) + ".mix.", a)) {
        if (!m40llm_ext_memory_serves(a.dim, a.dim)) throw std::invalid_argument("layer " + std::to_string(index) + ": head sizes beyond what the recurrence's kernels serve");
        const uint32_t cols = a.heads * a.dim;
        o_pad_ = round_up(cols, 32);
        ld_low_ = round_up(cols, 16);
        const size_t row = (size_t)rt.d_pad * 4, slot = m40llm_ext_channel_delta_state_floats(a.dim, a.dim) * a.heads * 4;
        last_row_ = rt.cleared(row * rt.opt.max_sequences);
        state_ = rt.cleared(slot * rt.opt.max_sequences);
        rt.states.push_back({&last_row_, row});
        rt.states.push_back({&state_, slot});
        rt.h_rows.want(rt.act_bytes(rt.d_pad));
        rt.proj.want(rt.f32_bytes((size_t)kSegments * w_->segment * 16));
        rt.cat.want(rt.act_bytes(o_pad_));
        sh_->mixes.want(rt.act_bytes((size_t)kMixes * rt.d_pad));
        sh_->low_act.want(rt.act_bytes(w_->low_pad));
        sh_->low.want(rt.f32_bytes(ld_low_));
        rt.want_planes(o_pad_ / 32, true);
    }
    bool reads_plain_rows() const override { return true; }
    void prepare(const Rows&) override { rows_.prepare(M40LLM_RULE_MIXING, a_.heads, a_.dim, a_.dim); }
    uint32_t enqueue(const Rows& r) override {
        const uint32_t d_tiles = rt_.d_pad / 32, ld = kSegments * w_->segment * 16, part = w_->segment * 16;
        {
            M40llmTokenMix m{};
            m.act_dtype = rt_.opt.act_dtype; m.rows = r.rows; m.ld = rt_.d_pad; m.mixes = kMixes;
            m.h = rt_.h_rows.ptr(); m.mu = w_->mu.ptr(); m.state = last_row_.ptr(); m.out = sh_->mixes.ptr();
            m.portions = rows_.portions().at; m.n_portions = rows_.portions().n; m.row_pos = r.pos; m.row_back = r.back;
            M40H_TRY(m40llm_ext_token_mix_async(rt_.ctx, &m, rt_.kStream));
        }
        {
            M40llmPackedGemm g = rt_.product(sh_->mixes.ptr(), kMixes * rt_.d_pad, w_->in, kSegments * w_->segment + w_->low_pad / 16, d_tiles, r.rows, M40LLM_PACKED_TANH);
            g.segment_tiles = w_->segment; g.a_batch = rt_.d_pad;
            g.plain_tiles = kSegments * w_->segment;
            g.out_f32 = rt_.proj.ptr(); g.ld_out = ld;
            g.out_act = sh_->low_act.ptr(); g.ld_act = w_->low_pad;
            rt_.launch(g);
        }
        {
            M40llmPackedGemm g = rt_.product(sh_->low_act.ptr(), w_->low_pad, w_->low, ld_low_ / 16, w_->low_pad / 32, r.rows, M40LLM_PACKED_STORE);
            g.out_f32 = sh_->low.ptr(); g.ld_out = ld_low_; g.cols = ld_low_;
            rt_.launch(g);
        }
        M40llmTimeMixing m{};
        m.act_dtype = rt_.opt.act_dtype; m.heads = a_.heads; m.dim = a_.dim;
        m.eps = rt_.spec.eps; m.out_factor = 1.0f;
        m.rkv = rt_.proj.ptr(); m.ld_rkv = ld;
        m.r_col = 0; m.k_col = part; m.v_col = 2 * part; m.g_col = 3 * part;
        m.decay = sh_->low.ptr(); m.ld_decay = ld_low_;
        m.w0 = w_->w0.ptr(); m.u = w_->u.ptr(); m.norm = w_->norm.ptr();
        m.state = state_.ptr();
        m.out = rt_.cat.ptr(); m.ld_out = o_pad_;
        rows_.enqueue(r, m, m40llm_ext_time_mixing_async);
        return rt_.into_planes(rt_.product(rt_.cat.ptr(), o_pad_, w_->out, round_up(rt_.spec.width, 16) / 16, o_pad_ / 32, r.rows, M40LLM_PACKED_STORE), r.rows);
    }

private:
    static constexpr uint32_t kSegments = 4, kMixes = 5;       // of the plain columns; of the tokens
    struct Weights {
        uint32_t segment, low_pad;         // column tiles of a plain part; padded rank of the decays
        DeviceBuf mu, in, low, w0, u, norm, out;
    };
    static std::shared_ptr<const Weights> load(LayerRuntime& rt, TensorSource& t, const std::string& p, const TimeMixingSpec& a) {
        const uint32_t D = rt.spec.width, d_tiles = rt.d_pad / 32, cols = a.heads * a.dim, rank = (uint32_t)t.rows_of(p + "w1", 64);
        auto w = std::make_shared<Weights>();
        w->low_pad = round_up(rank, 32);
        w->segment = round_up(std::max(round_up(cols, 16), w->low_pad) / 16, 16);
        w->in = rt.packed(kSegments * w->segment + w->low_pad / 16, d_tiles);
        std::vector<float> mu((size_t)kMixes * rt.d_pad, 0.0f);
        const char* names[kMixes] = {"r", "k", "v", "g", "w"};
        for (uint32_t i = 0; i < kMixes; ++i) {
            const std::vector<float> m = t.read_f32(p + "mu." + names[i], {D});
            std::copy(m.begin(), m.end(), mu.begin() + (size_t)i * rt.d_pad);
            if (i < kSegments) rt.pack(t, p + names[i], cols, D, w->in.ptr(), d_tiles, i * w->segment);
        }
        rt.pack(t, p + "w1", rank, D, w->in.ptr(), d_tiles, kSegments * w->segment);
        w->mu = rt.upload_f32(mu);
        w->low = rt.packed(round_up(cols, 16) / 16, w->low_pad / 32);
        rt.pack(t, p + "w2", cols, rank, w->low.ptr(), w->low_pad / 32, 0);
        w->w0 = rt.upload_f32(t.read_f32(p + "w0", {cols}));
        w->u = rt.upload_f32(t.read_f32(p + "u", {a.heads, a.dim}));
        w->norm = rt.upload_f32(t.read_f32(p + "norm", {cols}));
        w->out = rt.packed(round_up(D, 16) / 16, round_up(cols, 32) / 32);
        rt.pack(t, p + "o", D, cols, w->out.ptr(), round_up(cols, 32) / 32, 0);
        return w;
    }
    LayerRuntime& rt_;
    std::shared_ptr<StreamShared> sh_;
    TimeMixingSpec a_;
    RecurrentRows rows_;
    std::shared_ptr<const Weights> w_;
    uint32_t o_pad_, ld_low_;
    DeviceBuf last_row_, state_;
};

// Launches: product (gate, values, keys, queries, step sizes) | convolution | (convolution state of longer portions) | recurrence (longer bf16 portions:
// step sizes, states, outputs) | gate and norm | product
class StateSpaceMixer : public Mixer {
public:
    StateSpaceMixer(LayerRuntime& rt, std::shared_ptr<StreamShared> shared, TensorSource& t, uint32_t index, const StateSpaceSpec& a, const StateSpaceMixer* twin)
        : rt_(rt), sh_(std::move(shared)), a_(a), inner_(a.heads * a.vdim), conv_cols_(inner_ + 2 * a.groups * a.state), conv_col_(round_up(inner_, 16)),
          step_col_(conv_col_ + round_up(conv_cols_, 16)), tiles_in_((step_col_ + round_up(a.heads, 16)) / 16),
          ld_heads_(2 * a.groups * round_up(a.state, 32) + a.heads * round_up(a.vdim, 32)), o_pad_(round_up(inner_, 32)), rows_(rt, *sh_),
          w_(twin ? twin->w_ : load(t, "l" + std::to_string(index) + ".mix.")) {
        if (!m40llm_ext_lightning_serves(a.state, a.vdim)) throw std::invalid_argument("layer " + std::to_string(index) + ": head sizes beyond what the recurrence's kernels serve");
        if (a.taps > 1) {
            const size_t slot = (size_t)(a.taps - 1) * round_up(conv_cols_, 4) * 4;
            conv_state_ = rt.cleared(slot * rt.opt.max_sequences);
            rt.states.push_back({&conv_state_, slot});
        }
        const size_t slot = (size_t)a.heads * a.state * round_up(a.vdim, 32) * 4;
        state_ = rt.cleared(slot * rt.opt.max_sequences);
        rt.states.push_back({&state_, slot});
        rt.proj.want(rt.f32_bytes((size_t)tiles_in_ * 16));
        rt.cat.want(rt.act_bytes(o_pad_));
        sh_->heads.want(rt.act_bytes(ld_heads_));
        sh_->recurrent.want(rt.f32_bytes(round_up(inner_, 4)));
        rt.want_planes(o_pad_ / 32, true);
    }
    void prepare(const Rows&) override { rows_.prepare(m40llm_ext_lightning_scratch_bytes(rows_.portions().n_chunks, a_.heads, a_.state, a_.vdim)); }
    uint32_t enqueue(const Rows& r) override {
        const uint32_t ld = tiles_in_ * 16, ld_conv = round_up(conv_cols_, 4), ld_o = round_up(inner_, 4);
        {
            M40llmPackedGemm g = rt_.product(rt_.h.ptr(), rt_.d_pad, w_->in, tiles_in_, rt_.d_pad / 32, r.rows, M40LLM_PACKED_STORE);
            g.out_f32 = rt_.proj.ptr(); g.ld_out = ld; g.cols = ld;
            rt_.launch(g);
        }
        {
            M40llmSpaceSplit s{};
            s.act_dtype = rt_.opt.act_dtype; s.rows = r.rows; s.heads = a_.heads; s.kv_heads = a_.groups; s.dim = a_.state; s.vdim = a_.vdim; s.taps = a_.taps;
            s.proj = rt_.proj.f32(conv_col_); s.ld_proj = ld;
            s.conv = w_->conv.ptr(); s.bias = w_->conv_bias.ptr();
            s.conv_state = conv_state_.ptr(); s.ld_state = ld_conv;
            s.out = sh_->heads.ptr(); s.ld_out = ld_heads_;
            s.row_slot = r.slot; s.row_pos = r.pos; s.row_back = r.back;
            M40H_TRY(m40llm_ext_space_split_async(rt_.ctx, &s, rt_.kStream));
        }
        if (a_.taps > 1 && r.multi_row_portions)
            M40H_TRY(m40llm_ext_conv_state_async(rt_.ctx, rt_.proj.f32(conv_col_), ld, conv_cols_, a_.taps, conv_state_.ptr(), ld_conv, rows_.multi(), r.pos,
                                                 r.multi_row_portions, rt_.kStream));
        M40llmLightning l{};
        l.act_dtype = rt_.opt.act_dtype; l.heads = a_.heads; l.dim = a_.state; l.vdim = a_.vdim; l.kv_heads = a_.groups;
        l.qkv = sh_->heads.ptr(); l.ld_qkv = ld_heads_;
        l.step_logits = rt_.proj.f32(step_col_); l.ld_step = ld;
        l.step_bias = w_->step_bias.ptr(); l.A_log = w_->A_log.ptr(); l.skip = w_->skip.ptr();
        l.state = state_.ptr(); l.o = sh_->recurrent.ptr(); l.ld_o = ld_o;
        rows_.enqueue(r, l, m40llm_ext_lightning_async);
        M40H_TRY(m40llm_ext_gate_group_norm_rows_async(rt_.ctx, sh_->recurrent.ptr(), ld_o, rt_.proj.ptr(), ld, w_->norm.ptr(), r.rows, inner_, a_.norm_groups, rt_.spec.eps,
                                                       rt_.cat.ptr(), o_pad_, rt_.opt.act_dtype, rt_.kStream));
        return rt_.into_planes(rt_.product(rt_.cat.ptr(), o_pad_, w_->out, round_up(rt_.spec.width, 16) / 16, o_pad_ / 32, r.rows, M40LLM_PACKED_STORE), r.rows);
    }

private:
    struct Weights { DeviceBuf in, conv, conv_bias, step_bias, A_log, skip, norm, out; };
    std::shared_ptr<const Weights> load(TensorSource& t, const std::string& p) {
        const uint32_t D = rt_.spec.width, d_tiles = rt_.d_pad / 32;
        auto w = std::make_shared<Weights>();
        w->in = rt_.packed(tiles_in_, d_tiles);
        const void* rows = rt_.stage(t, p + "in", {(uint64_t)inner_ + conv_cols_ + a_.heads, D});
        rt_.pack_rows(rows, 0, inner_, D, w->in.ptr(), d_tiles, 0);
        rt_.pack_rows(rows, inner_, conv_cols_, D, w->in.ptr(), d_tiles, conv_col_ / 16);
        rt_.pack_rows(rows, inner_ + conv_cols_, a_.heads, D, w->in.ptr(), d_tiles, step_col_ / 16);
        w->conv = rt_.upload_taps(t, p + "conv", conv_cols_, a_.taps);
        w->conv_bias = rt_.upload_f32(t.read_f32(p + "conv.b", {conv_cols_}));
        w->step_bias = rt_.upload_f32(t.read_f32(p + "dt_bias", {a_.heads}));
        w->A_log = rt_.upload_f32(t.read_f32(p + "A_log", {a_.heads}));
        w->skip = rt_.upload_f32(t.read_f32(p + "D", {a_.heads}));
        w->norm = rt_.upload_f32(t.read_f32(p + "norm", {inner_}));
        w->out = rt_.packed(round_up(D, 16) / 16, o_pad_ / 32);
        rt_.pack(t, p + "o", D, inner_, w->out.ptr(), o_pad_ / 32, 0);
        return w;
    }
    LayerRuntime& rt_;
    std::shared_ptr<StreamShared> sh_;
    StateSpaceSpec a_;
    uint32_t inner_, conv_cols_, conv_col_, step_col_, tiles_in_, ld_heads_, o_pad_;
    RecurrentRows rows_;
    std::shared_ptr<const Weights> w_;
    DeviceBuf conv_state_, state_;
};

}  // namespace m40host
