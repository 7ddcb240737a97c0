// Decoder that runs a DecoderSpec: bf16 weights in packed tiles, bf16 or f32 activations, an f32 residual stream, a paged cache and, per
// sequence slot, what recurrent layers carry from token to token.  One step function takes any mixture of sequences and portions (whole
// prompts, parts of prompts, single tokens); everything that serves or generates goes through it or through the same layer launches
// replayed from a graph.  The layers themselves: latent_layer.hpp (parallel blocks), output_norm_layer.hpp, stream_layer.hpp, prenorm_layer.hpp.
#pragma once

#include <algorithm>
#include <chrono>
#include <cmath>
#include <cstring>
#include <map>
#include <memory>
#include <string>
#include <vector>

#include "latent_layer.hpp"
#include "output_norm_layer.hpp"
#include "stream_layer.hpp"
#include "prenorm_layer.hpp"
#include "served_model.hpp"

namespace m40host {

struct StepEntry {
    uint32_t sequence;
    const uint32_t* tokens;
    uint32_t n;
    const uint32_t* want;              // places among the tokens whose logits are asked for
    uint32_t n_want;
};

// Greedy picks of a step's wanted places, in the order of its logits rows: a row flagged greedy whose two best logits are no near
// tie is decided on the device (picks, picked = 1), and its logits are not brought back.
struct StepPicks {
    const uint8_t* greedy;
    uint32_t* picks;
    uint8_t* picked;
};

class LayeredDecoder : public ServedModel {
public:
    static constexpr uint32_t kStream = LayerRuntime::kStream;
    static constexpr uint32_t kPage = LayerRuntime::kPage;

    LayeredDecoder(M40llmCudaContext* ctx, DecoderSpec spec, TensorSource& tensors, const LayeredOptions& opt)
        : ctx_(ctx), spec_(std::move(spec)), opt_(checked(ctx, opt)), seqs_(round_up(opt.max_tokens, kPage) / kPage, kPage, opt.max_sequences),
          rt_(ctx, spec_, opt_, seqs_.total_pages()) {
        load(tensors);
        allocate();
    }
    ~LayeredDecoder() override {
        (void)m40llm_stream_synchronize(ctx_, kStream);
        drop_graph();
    }
    LayeredDecoder(const LayeredDecoder&) = delete;
    LayeredDecoder& operator=(const LayeredDecoder&) = delete;

    const DecoderSpec& spec() const { return spec_; }
    const SequencePages& sequences() const { return seqs_; }
    M40llmCudaContext* ctx() const { return ctx_; }

    const char* family() const override { return spec_.architecture.c_str(); }
    uint32_t vocab() const override { return spec_.vocab; }
    uint32_t max_seq_len() const override {
        const uint32_t pool = seqs_.total_pages() * kPage;
        return spec_.positions ? std::min(pool, spec_.positions) : pool;
    }
    uint32_t max_sequences() const override { return opt_.max_sequences; }
    void set_mode(uint32_t mode) override { mode_ = mode; drop_graph(); }
    void set_tie_guard(float g) override { tie_guard_ = g; }
    bool last_timed_host_fallback() const override { return timed_fallback_; }

    // gives back what a sequence holds
    void release(uint32_t seq) { seqs_.release(seq); }

    // Runs the entries' tokens behind what their sequences hold.  logits_out: [all wanted places, in entry order][vocab].
    // on_layer (optional): called after every layer with the rows of the pass and the residual on the device (diagnosis).
    void step(const std::vector<StepEntry>& entries, float* logits_out,
              const std::function<void(uint32_t layer, uint32_t rows, const float* x)>& on_layer = nullptr, const StepPicks* picks = nullptr) {
        std::vector<uint8_t> seen(opt_.max_sequences, 0);
        for (const auto& e : entries) {
            if (e.sequence >= opt_.max_sequences) throw std::out_of_range("sequence slot out of range");
            if (seen[e.sequence]++) throw std::invalid_argument("a sequence appears twice in a step");
            if (e.n == 0 || !e.tokens) throw std::invalid_argument("an entry has no tokens");
            for (uint32_t i = 0; i < e.n; ++i)
                if (e.tokens[i] >= spec_.vocab) throw std::out_of_range("token id out of range");
            for (uint32_t i = 0; i < e.n_want; ++i)
                if (e.want[i] >= e.n) throw std::out_of_range("a wanted place lies outside the entry's tokens");
            check_positions(e.sequence, e.n);
        }
        for (const auto& e : entries) seqs_.grow(e.sequence, (uint64_t)seqs_.length(e.sequence) + e.n);
        // passes of at most max_rows rows; an entry's rows stay in order
        std::vector<size_t> logits_at;       // first logits row of each entry
        size_t n_logits = 0;
        for (const auto& e : entries) { logits_at.push_back(n_logits); n_logits += e.n_want; }
        std::vector<uint32_t> done(entries.size(), 0);
        size_t first = 0;
        while (first < entries.size()) {
            struct Piece { size_t entry; uint32_t n; bool is_long; };
            std::vector<Piece> pieces;
            uint32_t taken = 0;
            for (size_t i = first; i < entries.size() && taken < opt_.max_rows; ++i) {
                const uint32_t n = std::min(entries[i].n - done[i], opt_.max_rows - taken);
                pieces.push_back({i, n, long_form(n, seqs_.length(entries[i].sequence))});
                taken += n;
            }
            // rows of single tokens and short portions come first
            std::stable_partition(pieces.begin(), pieces.end(), [](const Piece& p) { return !p.is_long; });
            PassPlan plan;
            for (const Piece& piece : pieces) {
                const size_t i = piece.entry;
                const StepEntry& e = entries[i];
                const uint32_t n = piece.n, len = seqs_.length(e.sequence);
                if (!piece.is_long) plan.short_rows += n;
                plan.portions.push_back({plan.rows(), n, e.sequence, len + n, piece.is_long});
                for (uint32_t k = 0; k < e.n_want; ++k)
                    if (e.want[k] >= done[i] && e.want[k] < done[i] + n) {
                        plan.want.push_back(plan.rows() + e.want[k] - done[i]);
                        plan.want_out.push_back(logits_at[i] + k);
                    }
                for (uint32_t k = 0; k < n; ++k) {
                    const uint32_t at = done[i] + k;
                    plan.tokens.push_back(e.tokens[at]);
                    plan.prev.push_back(at ? e.tokens[at - 1] : seqs_.previous_token(e.sequence));
                    plan.slot.push_back(e.sequence);
                    plan.pos.push_back(len + k);
                    plan.back.push_back(n == 1 ? kOnlyRow : k);
                }
                seqs_.advance(e.sequence, n, e.tokens[done[i] + n - 1]);
                done[i] += n;
            }
            while (first < entries.size() && done[first] == entries[first].n) ++first;
            run_pass(plan, logits_out, on_layer, picks);
        }
        M40H_TRY(m40llm_stream_synchronize(ctx_, kStream));
    }

    SchedulerEngine scheduler_engine() override {
        SchedulerEngine e;
        e.vocab = spec_.vocab;
        e.max_seq_len = max_seq_len();
        e.prefill = [this](const std::vector<SchedulerPrefillItem>& items, float* logits_out) {
            std::vector<SchedulerStepItem> s;
            for (const auto& it : items) s.push_back({it.sequence_id, 0, it.tokens, it.len, true});
            run_items(s, logits_out);
        };
        e.decode = [this](const std::vector<SchedulerDecodeItem>& items, float* logits_out) {
            std::vector<SchedulerStepItem> s;
            for (const auto& it : items) s.push_back({it.sequence_id, it.kv_len, &it.token, 1, true});
            run_items(s, logits_out);
        };
        e.step = [this](const std::vector<SchedulerStepItem>& items, const uint8_t* greedy, float* logits_out, uint32_t* picks, uint8_t* picked) {
            const StepPicks p{greedy, picks, picked};
            run_items(items, logits_out, mode_ >= 1 ? &p : nullptr);
        };
        e.reserve = [this](uint32_t seq, uint64_t tokens) { return seqs_.reserve(seq, tokens); };
        e.release = [this](uint32_t seq) { seqs_.release(seq); };
        e.step_tokens = opt_.max_rows;
        return e;
    }

    void decode_greedy(uint32_t seq, const uint32_t* prompt, uint32_t n_prompt, uint32_t n_gen, uint32_t start_pos, uint32_t* ids_out,
                       float* gaps_out) override {
        if (n_prompt == 0) throw std::invalid_argument("decode_greedy needs at least one prompt token");
        if (start_pos == 0) seqs_.release(seq);
        if (seqs_.length(seq) != start_pos) throw std::invalid_argument("the sequence does not hold start_pos tokens");
        std::vector<float> logits(spec_.vocab);
        std::copy(prompt, prompt + n_prompt, ids_out);
        const uint32_t last = n_prompt - 1;
        step({{seq, prompt, n_prompt, &last, n_gen ? 1u : 0u}}, logits.data());
        if (n_gen == 0) return;
        Sampler sampler = greedy_sampler(42);
        uint32_t next = (uint32_t)sampler.sample(logits.data(), logits.size());
        if (gaps_out) gaps_out[0] = DecodeModel::top2_gap(logits);
        ids_out[n_prompt] = next;
        if (n_gen == 1) return;
        const uint32_t len = seqs_.length(seq);
        decode_batch_greedy(&seq, &len, &next, 1, n_gen - 1, ids_out + n_prompt + 1, gaps_out ? gaps_out + 1 : nullptr);
    }

    void decode_batch_greedy(const uint32_t* seq_ids, const uint32_t* kv_lens, const uint32_t* first_tokens, uint32_t rows, uint32_t steps,
                             uint32_t* ids_out, float* gaps_out) override {
        generate(seq_ids, kv_lens, first_tokens, rows, 0, steps, ids_out, gaps_out, nullptr);
    }
    void decode_batch_timed(const uint32_t* seq_ids, const uint32_t* kv_lens, const uint32_t* first_tokens, uint32_t rows, uint32_t warmup,
                            uint32_t steps, uint32_t* ids_out, double* elapsed_ms) override {
        generate(seq_ids, kv_lens, first_tokens, rows, warmup, steps, ids_out, nullptr, elapsed_ms);
    }

    // Throughput runs: the sequence counts as holding `tokens` tokens whose entries are whatever its pages contain.
    void assume_length(uint32_t seq, uint32_t tokens) {
        seqs_.release(seq);
        seqs_.grow(seq, tokens);
        seqs_.advance(seq, tokens, 0);
    }

private:
    static constexpr uint32_t kOnlyRow = 0x80000000u;      // a portion of one row

    static LayeredOptions checked(M40llmCudaContext* ctx, LayeredOptions o) {
        if (!ctx) throw std::invalid_argument("null context");
        if (o.act_dtype > 1u || o.max_tokens == 0 || o.max_sequences == 0 || o.max_rows == 0) throw std::invalid_argument("bad model options");
        o.max_rows = std::min(o.max_rows, round_up(o.max_tokens, kPage));
        return o;
    }
    void check_positions(uint32_t seq, uint64_t more) const {
        if (spec_.positions && seqs_.length(seq) + more > spec_.positions) throw std::out_of_range("more tokens than the model has positions");
    }

    void load(TensorSource& t) {
        const uint32_t D = spec_.width, d_tiles = rt_.d_pad / 32;
        auto table = [&](const char* name, uint64_t rows) {
            DeviceBuf b(ctx_, rows * D * 2);
            t.read_bf16(ctx_, name, {rows, D}, b.ptr());
            return b;
        };
        embed_ = table("embed", spec_.vocab);
        if (spec_.bigram) bigram_ = table("bigram", (uint64_t)spec_.bigram->buckets + 1);
        if (spec_.positions) positions_ = table("pos", spec_.positions);
        switch (spec_.block) {
            case BlockKind::Parallel: load_parallel(t); break;
            case BlockKind::OutputNorm: load_output_norm(t); break;
            case BlockKind::Streams: load_streams(t); break;
            case BlockKind::PreNorm: load_pre_norm(t); break;
        }
        final_norm_ = rt_.upload_norm(t, "final.norm");
        head_ = rt_.packed(round_up(spec_.vocab, 16) / 16, d_tiles);
        rt_.pack(t, spec_.tied_head ? "embed" : "head", spec_.vocab, D, head_.ptr(), d_tiles, 0);
        rt_.finish_loading();
    }
    void load_parallel(TensorSource& t) {
        auto shared = std::make_shared<LatentShared>();
        shared_ = {shared};
        rt_.scratch.insert(rt_.scratch.end(), {&shared->cq, &shared->q, &shared->qa, &shared->ol});
        shared->per_head_served = rt_.bf16() && opt_.portion_form != 1u;
        for (const LayerSpec& s : spec_.layers) {
            const LatentAttentionSpec& a = std::get<LatentAttentionSpec>(s.mixer);
            shared->per_head_served = shared->per_head_served && m40llm_ext_head_attention_serves((round_up(a.dim, 32) + round_up(a.rot_dim, 32)) / 32, round_up(a.vdim, 16) / 16);
        }
        std::vector<LatentLayer*> made;
        for (const LayerSpec& s : spec_.layers) {
            const int from = std::get<LatentAttentionSpec>(s.mixer).kv_from;
            auto l = std::make_unique<LatentLayer>(rt_, shared, t, (uint32_t)made.size(), s, from >= 0 ? made[(size_t)from] : nullptr);
            made.push_back(l.get());
            layers_.push_back(std::move(l));
        }
    }
    void load_output_norm(TensorSource& t) {
        auto pair = std::make_shared<PairShared>();
        auto light = std::make_shared<LightningShared>();
        auto expert = std::make_shared<ExpertShared>();
        rt_.scratch.insert(rt_.scratch.end(), {&pair->queries, &light->qkv, &light->o, &expert->logits, &expert->ids, &expert->weight, &expert->rows_of,
                                               &expert->place, &expert->jobs, &expert->rows, &expert->act, &expert->out});
        shared_ = {pair, light, expert};
        std::vector<DifferentialMixer*> made;
        for (const LayerSpec& s : spec_.layers) {
            const uint32_t i = (uint32_t)made.size();
            std::unique_ptr<Mixer> mixer;
            made.push_back(nullptr);
            if (const auto* a = std::get_if<DifferentialAttentionSpec>(&s.mixer)) {
                auto m = std::make_unique<DifferentialMixer>(rt_, pair, t, i, *a, a->kv_from >= 0 ? made[(size_t)a->kv_from] : nullptr);
                made[i] = m.get();
                mixer = std::move(m);
            } else if (const auto* a = std::get_if<LightningSpec>(&s.mixer)) {
                mixer = std::make_unique<LightningMixer>(rt_, light, t, i, *a);
            } else {
                throw std::invalid_argument("layer " + std::to_string(i) + ": this mixer has no form with a norm on its output");
            }
            layers_.push_back(std::make_unique<OutputNormLayer>(rt_, t, i, std::move(mixer), feed_forward(t, expert, tensor_prefix(i), s.mlp)));
        }
    }
    void load_streams(TensorSource& t) {
        if (spec_.streams > M40LLM_MOST_STREAMS) throw std::invalid_argument("more residual streams than the kernels serve");
        auto shared = std::make_shared<StreamShared>();
        auto expert = std::make_shared<ExpertShared>();
        rt_.scratch.insert(rt_.scratch.end(), {&shared->queries, &shared->first_values, &shared->recurrent, &shared->low, &shared->low_act, &expert->logits, &expert->ids,
                                               &expert->weight, &expert->rows_of, &expert->place, &expert->jobs, &expert->rows, &expert->act, &expert->out});
        shared_ = {shared, expert};
        streams_ = std::make_unique<ResidualStreams>(rt_);
        bool values_kept = false;
        for (const LayerSpec& s : spec_.layers) {
            const uint32_t i = (uint32_t)layers_.size();
            std::unique_ptr<Mixer> mixer;
            if (const auto* a = std::get_if<AttentionSpec>(&s.mixer)) {
                mixer = std::make_unique<AttentionMixer>(rt_, shared, t, i, *a, a->share_values && values_kept);
                values_kept = values_kept || a->share_values;
            } else if (const auto* a = std::get_if<ParallelSpec>(&s.mixer)) {
                mixer = std::make_unique<ParallelMixer>(rt_, shared, t, i, *a);
            } else if (const auto* a = std::get_if<ChannelDeltaSpec>(&s.mixer)) {
                mixer = std::make_unique<ChannelDeltaMixer>(rt_, shared, t, i, *a);
            } else {
                throw std::invalid_argument("layer " + std::to_string(i) + ": this mixer has no form over residual streams");
            }
            if (const auto* e = std::get_if<ExpertMlpSpec>(&s.mlp); e && e->identity)
                throw std::invalid_argument("layer " + std::to_string(i) + ": experts that return their input have no form over residual streams");
            layers_.push_back(std::make_unique<StreamLayer>(rt_, *streams_, t, i, std::move(mixer), feed_forward(t, expert, tensor_prefix(i), s.mlp)));
        }
    }
    // Layers over one stream; those that use another layer's tensors (in whichever order the two come) share them and have a cache or state of
    // their own.
    void load_pre_norm(TensorSource& t) {
        auto shared = std::make_shared<StreamShared>();
        auto expert = std::make_shared<ExpertShared>();
        rt_.scratch.insert(rt_.scratch.end(), {&shared->queries, &shared->recurrent, &shared->low, &shared->low_act, &shared->mixes, &shared->heads, &expert->logits, &expert->ids,
                                               &expert->weight, &expert->rows_of, &expert->place, &expert->jobs, &expert->rows, &expert->act, &expert->out,
                                               &expert->slot_weight});
        shared_ = {shared, expert};
        streams_ = std::make_unique<ResidualStreams>(rt_);
        std::map<uint32_t, const StreamLayer*> made;        // by the layer whose tensors it has
        for (const LayerSpec& s : spec_.layers) {
            const uint32_t i = (uint32_t)layers_.size(), own = s.tensors_of >= 0 ? (uint32_t)s.tensors_of : i;
            const StreamLayer* twin = made.count(own) ? made[own] : nullptr;
            const Mixer* other = twin ? twin->mixer() : nullptr;
            std::unique_ptr<Mixer> mixer;
            if (const auto* a = std::get_if<AttentionSpec>(&s.mixer)) {
                mixer = std::make_unique<AttentionMixer>(rt_, shared, t, own, *a, false, dynamic_cast<const AttentionMixer*>(other));
            } else if (const auto* a = std::get_if<TimeMixingSpec>(&s.mixer)) {
                mixer = std::make_unique<TimeMixingMixer>(rt_, shared, t, own, *a, dynamic_cast<const TimeMixingMixer*>(other));
            } else if (const auto* a = std::get_if<StateSpaceSpec>(&s.mixer)) {
                mixer = std::make_unique<StateSpaceMixer>(rt_, shared, t, own, *a, dynamic_cast<const StateSpaceMixer*>(other));
            } else {
                throw std::invalid_argument("layer " + std::to_string(i) + ": this mixer has no pre-norm form");
            }
            auto layer = twin ? std::make_unique<StreamLayer>(*twin, std::move(mixer))
                              : std::make_unique<StreamLayer>(rt_, *streams_, t, own, std::move(mixer), feed_forward(t, expert, tensor_prefix(own), s.mlp));
            if (!twin) made[own] = layer.get();
            layers_.push_back(std::move(layer));
        }
    }
    static std::string tensor_prefix(uint32_t layer) { return "l" + std::to_string(layer) + "."; }
    std::unique_ptr<FeedForward> feed_forward(TensorSource& t, const std::shared_ptr<ExpertShared>& expert, const std::string& layer, const MlpSpec& mlp) {
        if (const auto* m = std::get_if<GatedMlpSpec>(&mlp)) return std::make_unique<DenseFeedForward>(rt_, t, layer, *m);
        if (const auto* m = std::get_if<PolyMlpSpec>(&mlp)) return std::make_unique<PolyFeedForward>(rt_, t, layer, *m);
        if (const auto* m = std::get_if<ExpertMlpSpec>(&mlp)) return std::make_unique<ExpertFeedForward>(rt_, expert, t, layer, *m);
        return nullptr;
    }

    void allocate() {
        rt_.allocate();
        logits_rows_ = std::min<uint32_t>(rt_.rows_pad, 256);
        hn_ = rt_.cleared((size_t)round_up(logits_rows_, 16) * rt_.d_pad * rt_.es);
        logits_ = DeviceBuf(ctx_, (size_t)logits_rows_ * spec_.vocab * 4);
        pick_parts_ = DeviceBuf(ctx_, (size_t)logits_rows_ * M40LLM_TOP2_PARTS * 16);
        for (const SlotState& s : rt_.states) state_bytes_ += s.slot_bytes;
        M40H_TRY(m40llm_stream_synchronize(ctx_, kStream));
    }

    // Whether the attention of a portion of n tokens behind `len` takes the form for long portions.
    bool long_form(uint32_t n, uint32_t len) const {
        if (!rt_.bf16() || opt_.portion_form == 1u || n == 1) return false;
        double as_tokens = 0.0, as_long = 0.0;
        for (const auto& l : layers_)
            if (!l->portion_cost(n, len, as_tokens, as_long)) return false;
        if (opt_.portion_form == 2u) return true;
        return n >= 32 && as_long < as_tokens;
    }

    void ensure_scratch(const Rows& r) {
        uint64_t need = 0;
        for (const auto& t : rt_.tables) need = std::max(need, t->partial_floats(r));
        for (const auto& l : layers_) l->prepare(r);
        if (need * 4 > rt_.partial.bytes()) {
            M40H_TRY(m40llm_stream_synchronize(ctx_, kStream));
            drop_graph();
            rt_.partial = DeviceBuf(ctx_, need * 4);
        }
    }
    std::vector<uint32_t> page_table() const {
        std::vector<uint32_t> t((size_t)opt_.max_sequences * rt_.max_pages, 0);
        for (uint32_t s = 0; s < opt_.max_sequences; ++s) std::copy(seqs_.pages(s).begin(), seqs_.pages(s).end(), t.begin() + (size_t)s * rt_.max_pages);
        return t;
    }
    // Uploads a plan's tables and gives their device addresses.
    Rows upload(const PassPlan& plan, DeviceBuf& buf, uint32_t longest, const uint32_t** want) {
        Rows r;
        r.rows = plan.rows();
        r.short_rows = plan.short_rows;
        for (const Portion& p : plan.portions) r.multi_row_portions += p.n > 1;
        std::vector<uint32_t> all;
        auto put = [&](const std::vector<uint32_t>& v) { const size_t at = all.size(); all.insert(all.end(), v.begin(), v.end()); return at; };
        const size_t tok = put(plan.tokens), prev = put(plan.prev), slot = put(plan.slot), pos = put(plan.pos), back = put(plan.back), w = put(plan.want),
                     table = put(page_table());
        std::vector<size_t> tables_at;
        for (auto& t : rt_.tables) tables_at.push_back(put(t->build(plan, seqs_, longest)));
        if (buf.bytes() < all.size() * 4) buf = DeviceBuf(ctx_, all.size() * 4 + all.size());
        M40H_TRY(m40llm_memcpy_h2d(ctx_, buf.ptr(), all.data(), all.size() * 4));
        r.tokens = buf.u32(tok); r.prev = buf.u32(prev); r.slot = buf.u32(slot); r.pos = buf.u32(pos); r.back = buf.u32(back); r.page_table = buf.u32(table);
        for (size_t i = 0; i < tables_at.size(); ++i) rt_.tables[i]->at = buf.u32(tables_at[i]);
        if (want) *want = buf.u32(w);
        return r;
    }

    void enqueue_embedding(const Rows& r) {
        rt_.pending = 0;
        const BigramSpec b = spec_.bigram.value_or(BigramSpec{});
        M40llmEmbedTokens e{};
        e.act_dtype = opt_.act_dtype; e.rows = r.rows; e.vocab = spec_.vocab; e.width = spec_.width;
        e.table = embed_.ptr(); e.pair_table = bigram_.ptr(); e.pos_table = positions_.ptr();
        e.tokens = r.tokens; e.prev = r.prev; e.positions = r.pos;
        e.buckets = b.buckets; e.mul_prev = b.mul_prev; e.mul_cur = b.mul_cur; e.n_positions = spec_.positions;
        e.scale = spec_.embedding_scale;
        e.x = rt_.x.ptr();
        if (spec_.block == BlockKind::OutputNorm) { e.h = rt_.h.ptr(); e.ld_h = rt_.d_pad; }
        M40H_TRY(m40llm_ext_embed_tokens_async(ctx_, &e, kStream));
        if (streams_) streams_->begin();
        for (auto& t : rt_.tables) t->enqueue(r);
    }
    // final norm and head of n of a pass's rows (row_index NULL = all of them)
    void enqueue_logits(const uint32_t* row_index, uint32_t n, uint32_t rows) {
        if (streams_) streams_->last_sum(row_index, n);
        M40H_TRY(m40llm_ext_norm_rows_async(ctx_, spec_.norm == NormKind::Rms ? M40LLM_NORM_RMS : M40LLM_NORM_LAYER, rt_.x.ptr(), rt_.planes.ptr(), rt_.pending,
                                            (uint64_t)rows * spec_.width, final_norm_.ptr(), row_index, n, spec_.width, spec_.eps, hn_.ptr(), rt_.d_pad,
                                            opt_.act_dtype, kStream));
        M40llmPackedGemm g = rt_.product(hn_.ptr(), rt_.d_pad, head_, round_up(spec_.vocab, 16) / 16, rt_.d_pad / 32, n, M40LLM_PACKED_STORE);
        if (spec_.logit_scale != 1.0f || spec_.logit_cap > 0.0f) {
            g.epilogue = M40LLM_PACKED_CAP;
            g.out_scale = spec_.logit_scale; g.out_cap = spec_.logit_cap;
        }
        g.out_f32 = logits_.ptr(); g.ld_out = spec_.vocab; g.cols = spec_.vocab;
        rt_.launch(g);
    }

    void run_pass(const PassPlan& plan, float* logits_out, const std::function<void(uint32_t, uint32_t, const float*)>& on_layer, const StepPicks* picks) {
        uint32_t longest = 0;
        for (const Portion& p : plan.portions)
            if (!p.is_long) longest = std::max(longest, p.length);
        M40H_TRY(m40llm_stream_synchronize(ctx_, kStream));           // the tables of the pass before may still be read
        const uint32_t* want = nullptr;
        Rows r = upload(plan, tables_, longest, &want);
        r.in_place = (bool)on_layer;
        ensure_scratch(r);
        enqueue_embedding(r);
        for (size_t i = 0; i < layers_.size(); ++i) {
            layers_[i]->enqueue(r);
            if (on_layer) {
                M40H_TRY(m40llm_stream_synchronize(ctx_, kStream));
                on_layer((uint32_t)i, r.rows, rt_.x.f32());
            }
        }
        for (size_t i = 0; i < plan.want.size(); i += logits_rows_) {
            const uint32_t n = (uint32_t)std::min<size_t>(logits_rows_, plan.want.size() - i);
            enqueue_logits(want + i, n, r.rows);
            std::vector<uint8_t> decided(n, 0);
            if (picks) {
                M40H_TRY(m40llm_ext_top2_parts_async(ctx_, logits_.ptr(), n, spec_.vocab, pick_parts_.ptr(), kStream));
                M40H_TRY(m40llm_stream_synchronize(ctx_, kStream));
                struct Part { float best, second; uint32_t at, unused; };
                std::vector<Part> parts((size_t)n * M40LLM_TOP2_PARTS);
                M40H_TRY(m40llm_memcpy_d2h(ctx_, parts.data(), pick_parts_.ptr(), parts.size() * sizeof(Part)));
                for (uint32_t k = 0; k < n; ++k) {
                    Part top = parts[(size_t)k * M40LLM_TOP2_PARTS];
                    for (uint32_t j = 1; j < M40LLM_TOP2_PARTS; ++j) {      // parts in order of their indices
                        const Part& p = parts[(size_t)k * M40LLM_TOP2_PARTS + j];
                        const bool take = p.best > top.best;
                        top.second = take ? std::max(top.best, p.second) : std::max(top.second, p.best);
                        if (take) { top.best = p.best; top.at = p.at; }
                    }
                    const size_t out = plan.want_out[i + k];
                    decided[k] = picks->greedy[out] && top.best - top.second >= tie_guard_ && top.at < spec_.vocab;
                    picks->picked[out] = decided[k];
                    picks->picks[out] = top.at;
                }
            }
            M40H_TRY(m40llm_stream_synchronize(ctx_, kStream));
            for (uint32_t k = 0; k < n;) {      // runs of rows that lie together in the output
                if (decided[k]) {
                    ++k;
                    continue;
                }
                uint32_t m = 1;
                while (k + m < n && !decided[k + m] && plan.want_out[i + k + m] == plan.want_out[i + k] + m) ++m;
                M40H_TRY(m40llm_memcpy_d2h(ctx_, logits_out + plan.want_out[i + k] * spec_.vocab, logits_.f32((size_t)k * spec_.vocab),
                                           (size_t)m * spec_.vocab * 4));
                k += m;
            }
        }
    }

    void run_items(const std::vector<SchedulerStepItem>& items, float* logits_out, const StepPicks* picks = nullptr) {
        std::vector<StepEntry> entries;
        std::vector<uint32_t> last(items.size());
        for (size_t i = 0; i < items.size(); ++i) {
            const SchedulerStepItem& it = items[i];
            if (it.start == 0 && seqs_.length(it.sequence_id) != 0) throw std::logic_error("the sequence slot was not given back");
            if (it.start != seqs_.length(it.sequence_id)) throw std::logic_error("the sequence does not hold the tokens before this portion");
            last[i] = it.len - 1;
            entries.push_back({it.sequence_id, it.tokens, it.len, &last[i], it.want ? 1u : 0u});
        }
        step(entries, logits_out, nullptr, picks);
    }

    // What recurrent layers carry for these slots, copied to (or back from) a buffer of its own.
    void copy_states(const uint32_t* slots, uint32_t n, bool back) {
        char* at = static_cast<char*>(state_copy_.ptr());
        for (const SlotState& s : rt_.states)
            for (uint32_t i = 0; i < n; ++i, at += s.slot_bytes) {
                char* own = static_cast<char*>(s.buf->ptr()) + slots[i] * s.slot_bytes;
                M40H_TRY(m40llm_memcpy_d2d_async(ctx_, back ? own : at, back ? at : own, s.slot_bytes, kStream));
            }
    }

    // Device-driven greedy steps: token, token before, position and step counter stay on the device.  Falls back to the host
    // sampler (states put back, same cache entries, rewritten) when a pick was a near tie.
    void generate(const uint32_t* seq_ids, const uint32_t* kv_lens, const uint32_t* first_tokens, uint32_t rows, uint32_t warmup, uint32_t steps,
                  uint32_t* ids_out, float* gaps_out, double* elapsed_ms) {
        const uint32_t total = warmup + steps;
        timed_fallback_ = false;
        if (rows == 0 || rows > opt_.max_sequences || rows > logits_rows_) throw std::invalid_argument("bad number of rows");
        if (total == 0) return;
        PassPlan plan;
        std::vector<uint32_t> len0(rows), prev0(rows);
        uint32_t longest = 0;
        for (uint32_t i = 0; i < rows; ++i) {
            const uint32_t s = seq_ids[i];
            if (seqs_.length(s) != kv_lens[i]) throw std::invalid_argument("a sequence does not hold the stated number of tokens");
            if (first_tokens[i] >= spec_.vocab) throw std::out_of_range("token id out of range");
            check_positions(s, total);
            seqs_.grow(s, (uint64_t)kv_lens[i] + total);
            len0[i] = kv_lens[i];
            prev0[i] = seqs_.previous_token(s);
            plan.tokens.push_back(first_tokens[i]);
            plan.prev.push_back(prev0[i]);
            plan.slot.push_back(s);
            plan.pos.push_back(kv_lens[i]);
            plan.back.push_back(kOnlyRow);
            plan.portions.push_back({i, 1, s, kv_lens[i] + 1, false});
            ++plan.short_rows;
            longest = std::max(longest, kv_lens[i] + total);
        }
        M40H_TRY(m40llm_stream_synchronize(ctx_, kStream));
        drop_graph();
        Rows r = upload(plan, loop_tables_, longest, nullptr);
        ensure_scratch(r);
        if (state_bytes_) {
            if (state_copy_.bytes() < state_bytes_ * rows) state_copy_ = DeviceBuf(ctx_, state_bytes_ * rows);
            copy_states(seq_ids, rows, false);
        }
        loop_state_ = rt_.cleared(16);
        loop_ids_ = DeviceBuf(ctx_, (size_t)rows * total * 4);
        loop_gaps_ = DeviceBuf(ctx_, (size_t)rows * total * 4);
        auto enqueue = [&]() {
            enqueue_embedding(r);
            for (auto& l : layers_) l->enqueue(r);
            enqueue_logits(nullptr, rows, rows);
            M40H_TRY(m40llm_ext_top2_parts_async(ctx_, logits_.ptr(), rows, spec_.vocab, pick_parts_.ptr(), kStream));
            M40H_TRY(m40llm_ext_advance_rows_async(ctx_, pick_parts_.ptr(), rows, r.tokens, r.prev, r.pos, loop_state_.u32(), loop_ids_.u32(),
                                                   loop_gaps_.f32(), total, kStream));
        };
        auto run = [&](uint32_t n) {
            if (mode_ >= 2 && n > 0) {
                if (!graph_) {
                    M40H_TRY(m40llm_stream_synchronize(ctx_, kStream));
                    M40H_TRY(m40llm_cuda_graph_begin_capture(ctx_, kStream));
                    try {
                        enqueue();
                    } catch (...) {
                        m40llm_cuda_graph_cancel_capture(ctx_, kStream);
                        throw;
                    }
                    M40H_TRY(m40llm_cuda_graph_end_capture(ctx_, kStream, &graph_));
                }
                for (uint32_t i = 0; i < n; ++i) M40H_TRY(m40llm_cuda_graph_launch(ctx_, graph_, kStream));
            } else {
                for (uint32_t i = 0; i < n; ++i) enqueue();
            }
        };
        run(warmup);
        M40H_TRY(m40llm_stream_synchronize(ctx_, kStream));
        const auto t0 = std::chrono::steady_clock::now();
        run(steps);
        M40H_TRY(m40llm_stream_synchronize(ctx_, kStream));
        const auto t1 = std::chrono::steady_clock::now();
        if (elapsed_ms) *elapsed_ms = std::chrono::duration<double, std::milli>(t1 - t0).count();
        std::vector<float> gaps((size_t)rows * total);
        M40H_TRY(m40llm_memcpy_d2h(ctx_, ids_out, loop_ids_.ptr(), (size_t)rows * total * 4));
        M40H_TRY(m40llm_memcpy_d2h(ctx_, gaps.data(), loop_gaps_.ptr(), gaps.size() * 4));
        drop_graph();
        bool ok = true;
        for (float g : gaps) ok = ok && g >= tie_guard_;
        if (ok) {
            for (uint32_t i = 0; i < rows; ++i) {
                const uint32_t* ids = ids_out + (size_t)i * total;
                seqs_.advance(seq_ids[i], total, total > 1 ? ids[total - 2] : first_tokens[i]);
            }
            if (gaps_out) std::copy(gaps.begin(), gaps.end(), gaps_out);
            return;
        }
        timed_fallback_ = true;
        if (state_bytes_) copy_states(seq_ids, rows, true);
        std::vector<uint32_t> tokens(first_tokens, first_tokens + rows);
        std::vector<float> logits((size_t)rows * spec_.vocab);
        std::vector<Sampler> samplers(rows, greedy_sampler(42));
        const uint32_t zero = 0;
        const auto h0 = std::chrono::steady_clock::now();
        auto h1 = h0;
        for (uint32_t s = 0; s < total; ++s) {
            if (s == warmup) h1 = std::chrono::steady_clock::now();
            std::vector<StepEntry> entries;
            for (uint32_t i = 0; i < rows; ++i) entries.push_back({seq_ids[i], &tokens[i], 1, &zero, 1});
            step(entries, logits.data());
            for (uint32_t i = 0; i < rows; ++i) {
                const float* l = logits.data() + (size_t)i * spec_.vocab;
                tokens[i] = (uint32_t)samplers[i].sample(l, spec_.vocab);
                ids_out[(size_t)i * total + s] = tokens[i];
                if (gaps_out) gaps_out[(size_t)i * total + s] = DecodeModel::top2_gap(l, spec_.vocab);
            }
        }
        if (elapsed_ms) *elapsed_ms = std::chrono::duration<double, std::milli>(std::chrono::steady_clock::now() - h1).count();
    }
    void drop_graph() {
        if (graph_) m40llm_cuda_graph_destroy(graph_);
        graph_ = nullptr;
    }

    M40llmCudaContext* ctx_;
    DecoderSpec spec_;
    LayeredOptions opt_;
    SequencePages seqs_;
    LayerRuntime rt_;
    uint32_t logits_rows_ = 0, mode_ = 2;
    float tie_guard_ = DecodeModel::kGreedyTieGuard;
    bool timed_fallback_ = false;
    std::vector<std::shared_ptr<void>> shared_;       // buffers the layers share
    std::unique_ptr<ResidualStreams> streams_;        // BlockKind::Streams, PreNorm
    std::vector<std::unique_ptr<DecoderLayer>> layers_;
    size_t state_bytes_ = 0;                          // of a slot, all layers
    DeviceBuf embed_, bigram_, positions_, final_norm_, head_, hn_, logits_, pick_parts_, tables_;
    DeviceBuf loop_tables_, loop_state_, loop_ids_, loop_gaps_, state_copy_;
    M40llmCudaGraphExec* graph_ = nullptr;
};

// A folder with config.json and model.safetensors.
inline std::unique_ptr<LayeredDecoder> open_model_folder(M40llmCudaContext* ctx, const std::string& dir, const LayeredOptions& opt) {
    DecoderSpec spec = read_decoder_spec(read_text_file(dir + "/config.json"));
    SafetensorsFile file(dir + "/model.safetensors");
    return std::make_unique<LayeredDecoder>(ctx, std::move(spec), file, opt);
}

}  // namespace m40host
