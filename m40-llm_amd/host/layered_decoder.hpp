// Decoder that runs a DecoderSpec: bf16 weights in packed tiles, bf16 or f32 activations, an f32 residual stream, a paged latent
// cache.  One step function takes any mixture of sequences and portions (whole prompts, parts of prompts, single tokens);
// everything that serves or generates goes through it or through the same layer launches replayed from a graph.
//
// Launches of a layer (all on the decode stream):
//   layer norm                      h = norm(x)
//   packed product, PROJECT         [q latent | kv latent | rotated key | gate logits] -> f32, gelu(gate) * up -> bf16
//   latent split                    norms of the two latents, key rotation, cache append
//   packed product, ROTATE          queries from their latent, rotated part turned in the last step
// then for the rows of decoded tokens and short portions
//   packed product per head         queries into latent space (W_uk^T)
//   latent attention (+ join)       over the pages, sink in the denominator
//   packed product per head, GATED  values from latent sums (W_uv), times the head's gate
// and for the rows of long portions, where bringing a sequence's keys and values out of the latents costs less than it saves
//   page products, KEYS and VALUES  the heads' keys and values of the portions' sequences
//   head attention                  causal, sink, times the head's gate
// and for all rows
//   packed product, ADD             x += [W_o | W_down] [attention ; feed-forward]; small launches store the sums of parts of K
//                                   instead, and the next norm adds them
#pragma once

#include <algorithm>
#include <chrono>
#include <cmath>
#include <cstring>
#include <memory>
#include <string>
#include <vector>

#include "decoder_spec.hpp"
#include "model.hpp"
#include "page_pool.hpp"
#include "safetensors.hpp"
#include "served_model.hpp"

namespace m40host {

inline uint32_t round_up(uint32_t n, uint32_t m) { return (n + m - 1) / m * m; }

struct LayeredOptions {
    uint32_t act_dtype = M40LLM_ACT_BF16;
    uint32_t max_tokens = 4096;        // what the cache pool holds, in tokens
    uint32_t max_sequences = 4;
    uint32_t max_rows = 4096;          // rows of one pass; longer steps run in several
    uint32_t portion_form = 0;         // attention of portions: 0 the cheaper, 1 in latent space, 2 head by head where it is served
};

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
    static constexpr uint32_t kStream = M40LLM_STREAM_DECODE;
    static constexpr uint32_t kPage = M40LLM_PAGE_TOKENS;
    static constexpr uint32_t kCus = 256, kMaxParts = 8;

    LayeredDecoder(M40llmCudaContext* ctx, DecoderSpec spec, TensorSource& tensors, const LayeredOptions& opt)
        : ctx_(ctx), spec_(std::move(spec)), opt_(opt), es_(opt.act_dtype == M40LLM_ACT_F32 ? 4u : 2u),
          seqs_(round_up(opt.max_tokens, kPage) / kPage, kPage, opt.max_sequences) {
        if (!ctx) throw std::invalid_argument("null context");
        if (opt.act_dtype > 1u || opt.max_tokens == 0 || opt.max_sequences == 0 || opt.max_rows == 0) throw std::invalid_argument("bad model options");
        opt_.max_rows = std::min(opt_.max_rows, round_up(opt.max_tokens, kPage));
        max_pages_ = seqs_.total_pages();
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
    uint32_t max_seq_len() const override { return seqs_.total_pages() * kPage; }
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
        }
        for (const auto& e : entries) seqs_.grow(e.sequence, (uint64_t)seqs_.length(e.sequence) + e.n);
        // passes of at most max_rows rows; an entry's rows stay in order
        std::vector<size_t> logits_at;       // first logits row of each entry
        size_t n_logits = 0;
        for (const auto& e : entries) { logits_at.push_back(n_logits); n_logits += e.n_want; }
        std::vector<uint32_t> done(entries.size(), 0);
        size_t first = 0;
        while (first < entries.size()) {
            struct Piece { size_t entry; uint32_t n; bool per_head; };
            std::vector<Piece> pieces;
            uint32_t taken = 0;
            for (size_t i = first; i < entries.size() && taken < opt_.max_rows; ++i) {
                const uint32_t n = std::min(entries[i].n - done[i], opt_.max_rows - taken);
                pieces.push_back({i, n, per_head(n, seqs_.length(entries[i].sequence))});
                taken += n;
            }
            // rows whose attention runs in latent space come first
            std::stable_partition(pieces.begin(), pieces.end(), [](const Piece& p) { return !p.per_head; });
            PassPlan plan;
            for (const Piece& piece : pieces) {
                const size_t i = piece.entry;
                const StepEntry& e = entries[i];
                const uint32_t n = piece.n, len = seqs_.length(e.sequence);
                if (!piece.per_head) plan.latent_rows += n;
                plan.portions.push_back({plan.rows(), n, e.sequence, len + n, piece.per_head});
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
    struct Layer {
        LatentAttentionSpec a;
        uint32_t ff = 0;                      // 0 = no feed-forward
        uint32_t dim_pad, rot_pad, q_width;   // a head's query: [dim_pad | rot_pad]
        uint32_t latent_pad, entry_width;
        uint32_t cq_pad;
        uint32_t plain_tiles, proj_tiles, kv_offset, rot_offset, gate_offset;
        uint32_t o_pad, ff_pad, cat;          // [attention | feed-forward] columns
        uint32_t vdim_tiles;
        int rotation;                         // index into rotations_
        int tile_set;                         // index into tile_sets_
        float scale;
        DeviceBuf norm1, w_proj, q_norm, kv_norm, w_uq, w_ukt, w_uk, w_uv, sink, w_out, cache;
    };
    struct Rotation {
        RotationSpec spec;
        uint32_t half;                        // padded pairs of a row
        DeviceBuf freq, angles;
    };
    struct TileSet {
        uint32_t heads, max_m_tiles, latent_pad;
    };
    struct Portion { uint32_t row, n, slot, length; bool per_head; };      // length: tokens its sequence holds at its end
    struct PassPlan {
        std::vector<uint32_t> tokens, prev, slot, pos, want;
        std::vector<size_t> want_out;
        std::vector<Portion> portions;
        uint32_t latent_rows = 0;
        uint32_t rows() const { return (uint32_t)tokens.size(); }
    };
    // device addresses of a pass
    struct Rows {
        uint32_t rows = 0;
        bool in_place = false;                // every layer leaves its result in x
        uint32_t *tokens = nullptr, *prev = nullptr, *slot = nullptr, *pos = nullptr, *page_table = nullptr;
        uint32_t latent_rows = 0;             // rows before it: attention in latent space; from it on: head by head
        const uint32_t *jobs = nullptr, *page_list = nullptr;
        uint32_t n_jobs = 0, job_rows = 128, n_pages = 0;
        struct Tiles { const uint32_t* table = nullptr; uint32_t n = 0, m_tiles = 1, splits = 1; };
        std::vector<Tiles> tiles;             // one per tile set
    };

    static DeviceBuf cleared(M40llmCudaContext* ctx, size_t bytes) {
        DeviceBuf b(ctx, (bytes + 15) / 16 * 16);
        M40H_TRY(m40llm_ext_clear_u32_async(ctx, b.ptr(), b.bytes() / 4, kStream));
        return b;
    }
    DeviceBuf upload_f32(const std::vector<float>& v) {
        DeviceBuf b(ctx_, v.size() * 4);
        M40H_TRY(m40llm_memcpy_h2d(ctx_, b.ptr(), v.data(), v.size() * 4));
        return b;
    }
    void* stage(TensorSource& t, const std::string& name, const std::vector<uint64_t>& shape) {
        const size_t bytes = tensor_elements(shape) * 2;
        M40H_TRY(m40llm_stream_synchronize(ctx_, kStream));       // the tensor before may still be being packed
        if (staging_.bytes() < bytes) staging_ = DeviceBuf(ctx_, bytes);
        t.read_bf16(ctx_, name, shape, staging_.ptr());
        return staging_.ptr();
    }
    static DeviceBuf packed(M40llmCudaContext* ctx, uint32_t n_tiles, uint32_t k_tiles) { return cleared(ctx, (size_t)n_tiles * k_tiles * 1024); }
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
        M40H_TRY(m40llm_ext_pack_tiles_async(ctx_, static_cast<const uint16_t*>(src) + (size_t)first * K, dst, &p, kStream));
    }
    // per head: rows [first, first + n) of the head's `stride` rows of [heads * stride][K] to packed rows offset .. of its block_pad
    void pack_heads(const void* src, uint32_t heads, uint32_t stride, uint32_t first, uint32_t n, uint32_t K, void* dst, uint32_t k_tiles,
                    uint32_t block_pad, uint32_t offset) {
        M40llmPackPlan p{};
        p.n_blocks = heads; p.n = n; p.n_block_pad = block_pad; p.n_offset = offset;
        p.k_blocks = 1; p.k = K; p.k_block_pad = K;
        p.sn_block = (uint64_t)stride * K; p.sn = K; p.sk = 1;
        p.k_tiles = k_tiles; p.tile_stride = 1;
        M40H_TRY(m40llm_ext_pack_tiles_async(ctx_, static_cast<const uint16_t*>(src) + (size_t)first * K, dst, &p, kStream));
    }

    void load(TensorSource& t) {
        per_head_served_ = opt_.act_dtype == M40LLM_ACT_BF16 && opt_.portion_form != 1u;
        for (const LayerSpec& s : spec_.layers)
            per_head_served_ = per_head_served_ && m40llm_ext_head_attention_serves((round_up(s.mixer.dim, 32) + round_up(s.mixer.rot_dim, 32)) / 32,
                                                                                    round_up(s.mixer.vdim, 16) / 16);
        const uint32_t D = spec_.width, d_tiles = round_up(D, 32) / 32;
        embed_ = DeviceBuf(ctx_, (size_t)spec_.vocab * D * 2);
        t.read_bf16(ctx_, "embed", {spec_.vocab, D}, embed_.ptr());
        if (spec_.bigram) {
            const uint64_t n = (uint64_t)spec_.bigram->buckets + 1;
            bigram_ = DeviceBuf(ctx_, n * D * 2);
            t.read_bf16(ctx_, "bigram", {n, D}, bigram_.ptr());
        }
        for (size_t i = 0; i < spec_.layers.size(); ++i) {
            const LayerSpec& s = spec_.layers[i];
            const std::string p = "l" + std::to_string(i) + ".", x = p + "mix.";
            layers_.emplace_back();
            Layer& l = layers_.back();
            l.a = s.mixer;
            l.ff = s.mlp ? s.mlp->ff : 0;
            const LatentAttentionSpec& a = l.a;
            const bool own = a.kv_from < 0;
            l.dim_pad = round_up(a.dim, 32); l.rot_pad = round_up(a.rot_dim, 32); l.q_width = l.dim_pad + l.rot_pad;
            l.latent_pad = round_up(a.kv_rank, 32); l.entry_width = l.latent_pad + l.rot_pad;
            l.cq_pad = round_up(a.q_rank, 32);
            l.kv_offset = round_up(a.q_rank, 16);
            l.rot_offset = l.kv_offset + (own ? round_up(a.kv_rank, 16) : 0);
            l.gate_offset = l.rot_offset + (own ? round_up(a.rot_dim, 16) : 0);
            l.plain_tiles = round_up(l.gate_offset + round_up(a.heads, 16), 32) / 16;
            l.proj_tiles = l.plain_tiles + 2 * (round_up(l.ff, 16) / 16);
            l.o_pad = round_up(a.heads * a.vdim, 32); l.ff_pad = round_up(l.ff, 32); l.cat = l.o_pad + l.ff_pad;
            l.vdim_tiles = round_up(a.vdim, 16) / 16;
            l.scale = a.scale;
            l.rotation = rotation_index(a.rotation, l.rot_pad / 2);
            const uint32_t max_m = m40llm_ext_latent_attention_max_m_tiles(opt_.act_dtype, a.kv_rank, l.entry_width);
            if (max_m == 0) throw std::invalid_argument("layer " + std::to_string(i) + ": kv_rank + rot_dim beyond what the attention kernels serve");
            l.tile_set = tile_set_index(a.heads, max_m, l.latent_pad);

            l.norm1 = upload_f32(t.read_f32(p + "norm1", {D}));
            l.q_norm = upload_f32(t.read_f32(x + "dq.norm", {a.q_rank}));
            l.sink = upload_f32(t.read_f32(x + "sink", {a.heads}));
            l.w_proj = packed(ctx_, l.proj_tiles, d_tiles);
            pack(t, x + "dq", a.q_rank, D, l.w_proj.ptr(), d_tiles, 0);
            if (own) {
                l.kv_norm = upload_f32(t.read_f32(x + "dkv.norm", {a.kv_rank}));
                const void* src = stage(t, x + "dkv", {a.kv_rank + a.rot_dim, D});
                pack_rows(src, 0, a.kv_rank, D, l.w_proj.ptr(), d_tiles, l.kv_offset / 16);
                pack_rows(src, a.kv_rank, a.rot_dim, D, l.w_proj.ptr(), d_tiles, l.rot_offset / 16);
            }
            pack(t, x + "g", a.heads, D, l.w_proj.ptr(), d_tiles, l.gate_offset / 16);
            if (l.ff) {
                pack(t, p + "mlp.gate", l.ff, D, l.w_proj.ptr(), d_tiles, l.plain_tiles, 0, 2);
                pack(t, p + "mlp.up", l.ff, D, l.w_proj.ptr(), d_tiles, l.plain_tiles + 1, 0, 2);
            }
            {
                const uint32_t kt = l.cq_pad / 32;
                l.w_uq = packed(ctx_, a.heads * l.q_width / 16, kt);
                const void* src = stage(t, x + "uq", {(uint64_t)a.heads * (a.dim + a.rot_dim), a.q_rank});
                pack_heads(src, a.heads, a.dim + a.rot_dim, 0, a.dim, a.q_rank, l.w_uq.ptr(), kt, l.q_width, 0);
                pack_heads(src, a.heads, a.dim + a.rot_dim, a.dim, a.rot_dim, a.q_rank, l.w_uq.ptr(), kt, l.q_width, l.dim_pad);
            }
            {   // W_uk [heads * dim][kv_rank] as one [kv_rank][dim] matrix a head
                l.w_ukt = packed(ctx_, a.heads * l.latent_pad / 16, l.dim_pad / 32);
                const void* src = stage(t, x + "uk", {(uint64_t)a.heads * a.dim, a.kv_rank});
                M40llmPackPlan q{};
                q.n_blocks = a.heads; q.n = a.kv_rank; q.n_block_pad = l.latent_pad;
                q.k_blocks = 1; q.k = a.dim; q.k_block_pad = a.dim;
                q.sn_block = (uint64_t)a.dim * a.kv_rank; q.sn = 1; q.sk = a.kv_rank;
                q.k_tiles = l.dim_pad / 32; q.tile_stride = 1;
                M40H_TRY(m40llm_ext_pack_tiles_async(ctx_, src, l.w_ukt.ptr(), &q, kStream));
                if (per_head_served_) {
                    l.w_uk = packed(ctx_, a.heads * l.dim_pad / 16, l.latent_pad / 32);
                    pack_heads(src, a.heads, a.dim, 0, a.dim, a.kv_rank, l.w_uk.ptr(), l.latent_pad / 32, l.dim_pad, 0);
                }
            }
            {
                const uint32_t kt = l.latent_pad / 32;
                l.w_uv = packed(ctx_, a.heads * l.vdim_tiles, kt);
                const void* src = stage(t, x + "uv", {(uint64_t)a.heads * a.vdim, a.kv_rank});
                pack_heads(src, a.heads, a.vdim, 0, a.vdim, a.kv_rank, l.w_uv.ptr(), kt, l.vdim_tiles * 16, 0);
            }
            l.w_out = packed(ctx_, round_up(D, 16) / 16, l.cat / 32);
            pack(t, x + "o", D, a.heads * a.vdim, l.w_out.ptr(), l.cat / 32, 0, 0);
            if (l.ff) pack(t, p + "mlp.down", D, l.ff, l.w_out.ptr(), l.cat / 32, 0, l.o_pad);
            if (own) l.cache = cleared(ctx_, (size_t)max_pages_ * kPage * l.entry_width * es_);
        }
        final_norm_ = upload_f32(t.read_f32("final.norm", {D}));
        head_ = packed(ctx_, round_up(spec_.vocab, 16) / 16, d_tiles);
        pack(t, "head", spec_.vocab, D, head_.ptr(), d_tiles, 0);
        M40H_TRY(m40llm_stream_synchronize(ctx_, kStream));
        staging_ = DeviceBuf();
    }
    int rotation_index(const RotationSpec& r, uint32_t half) {
        for (size_t i = 0; i < rotations_.size(); ++i)
            if (rotations_[i].spec == r && rotations_[i].half == half) return (int)i;
        Rotation n;
        n.spec = r;
        n.half = half;
        const std::vector<double> f = r.frequencies();
        n.freq = DeviceBuf(ctx_, std::max<size_t>(f.size(), 1) * 8);
        if (!f.empty()) M40H_TRY(m40llm_memcpy_h2d(ctx_, n.freq.ptr(), f.data(), f.size() * 8));
        rotations_.push_back(std::move(n));
        return (int)rotations_.size() - 1;
    }
    int tile_set_index(uint32_t heads, uint32_t max_m, uint32_t latent_pad) {
        for (size_t i = 0; i < tile_sets_.size(); ++i)
            if (tile_sets_[i].heads == heads && tile_sets_[i].max_m_tiles == max_m && tile_sets_[i].latent_pad == latent_pad) return (int)i;
        tile_sets_.push_back({heads, max_m, latent_pad});
        return (int)tile_sets_.size() - 1;
    }

    void allocate() {
        const size_t R = round_up(std::max(opt_.max_rows, opt_.max_sequences), 16), D = spec_.width;
        size_t proj = 0, cat = 0, cq = 0, q = 0, qa = 0, ol = 0;
        for (const Layer& l : layers_) {
            proj = std::max<size_t>(proj, (size_t)l.plain_tiles * 16);
            cat = std::max<size_t>(cat, l.cat);
            cq = std::max<size_t>(cq, l.cq_pad);
            q = std::max<size_t>(q, (size_t)l.a.heads * l.q_width);
            qa = std::max<size_t>(qa, (size_t)l.a.heads * l.entry_width);
            ol = std::max<size_t>(ol, (size_t)l.a.heads * l.latent_pad);
        }
        d_pad_ = round_up((uint32_t)D, 32);
        x_ = cleared(ctx_, R * D * 4);
        size_t planes = 0;         // most floats the parts of a step's sums take
        for (uint32_t rows = 1; rows <= R; ++rows)
            for (const Layer& l : layers_) {
                const uint32_t parts = k_parts(round_up((uint32_t)D, 16) / 16, l.cat / 32, rows);
                if (parts > 1) planes = std::max<size_t>(planes, (size_t)parts * rows * D);
            }
        planes_ = DeviceBuf(ctx_, std::max<size_t>(planes, 4) * 4);
        h_ = cleared(ctx_, R * d_pad_ * es_);
        proj_ = cleared(ctx_, R * proj * 4);
        cat_ = cleared(ctx_, R * cat * es_);
        cq_ = cleared(ctx_, R * cq * es_);
        q_ = cleared(ctx_, R * q * es_);
        qa_ = cleared(ctx_, R * qa * es_);
        ol_ = cleared(ctx_, R * ol * es_);
        for (Rotation& r : rotations_) r.angles = cleared(ctx_, R * r.half * 8);
        logits_rows_ = (uint32_t)std::min<size_t>(std::max<size_t>(R, opt_.max_sequences), 256);
        hn_ = cleared(ctx_, (size_t)round_up(logits_rows_, 16) * d_pad_ * es_);
        logits_ = DeviceBuf(ctx_, (size_t)logits_rows_ * spec_.vocab * 4);
        pick_parts_ = DeviceBuf(ctx_, (size_t)logits_rows_ * M40LLM_TOP2_PARTS * 16);
        M40H_TRY(m40llm_stream_synchronize(ctx_, kStream));
    }

    // Whether a portion of n tokens behind `len` takes the attention head by head: two products over every pair of a query and a key it
    // sees, against bringing all keys and values out of the latents first.  The latent form's kernel reaches half the rate.
    bool per_head(uint32_t n, uint32_t len) const {
        if (!per_head_served_ || n == 1) return false;
        if (opt_.portion_form == 2u) return true;
        if (n < 32) return false;
        double latent = 0.0, head = 0.0;
        const double keys = (double)len + n, seen = (double)n * (len + n / 2.0);
        for (const Layer& l : layers_) {
            latent += 2.0 * seen * l.a.heads * (l.entry_width + l.latent_pad) + (double)n * l.a.heads * l.latent_pad * (l.dim_pad + l.a.vdim);
            head += seen * l.a.heads * (l.q_width + l.a.vdim) + keys * l.a.heads * l.latent_pad * (l.dim_pad + l.a.vdim);
        }
        return head < latent;
    }

    // query tiles of a set for the portions of a pass
    static void make_tiles(const TileSet& set, const std::vector<Portion>& portions, std::vector<uint32_t>& table, uint32_t& m_tiles) {
        uint32_t longest = 0;
        for (const Portion& p : portions)
            if (!p.per_head) longest = std::max(longest, p.n * set.heads);
        m_tiles = longest <= 16 ? 1 : longest <= 32 ? 2 : 4;
        m_tiles = std::min(m_tiles, set.max_m_tiles);
        const uint32_t size = 16 * m_tiles;
        for (const Portion& p : portions)
            for (uint32_t i = 0; !p.per_head && i < p.n * set.heads; i += size) {
                table.push_back(p.row * set.heads + i);
                table.push_back(std::min(size, p.n * set.heads - i));
            }
    }
    static uint32_t choose_splits(uint32_t n_tiles, uint32_t longest) {
        const uint32_t pages = (longest + kPage - 1) / kPage;
        return std::max(1u, std::min(pages, 256u / std::max(n_tiles, 1u)));
    }
    void ensure_scratch(const Rows& r) {
        uint64_t need = 0;
        for (size_t i = 0; i < tile_sets_.size(); ++i)
            need = std::max(need, m40llm_ext_latent_attention_partial_floats(r.latent_rows * tile_sets_[i].heads, tile_sets_[i].latent_pad, r.tiles[i].splits));
        uint64_t keys = 0, values = 0;
        for (const Layer& l : layers_) {
            keys = std::max(keys, (uint64_t)r.n_pages * kPage * l.a.heads * l.dim_pad * 2);
            values = std::max(values, (uint64_t)r.n_pages * kPage * l.a.heads * l.vdim_tiles * 16 * 2);
        }
        if (keys > keys_.bytes() || values > values_.bytes()) {
            M40H_TRY(m40llm_stream_synchronize(ctx_, kStream));
            keys_ = DeviceBuf(ctx_, keys);
            values_ = DeviceBuf(ctx_, values);
        }
        if (need * 4 > partial_.bytes()) {
            M40H_TRY(m40llm_stream_synchronize(ctx_, kStream));
            drop_graph();
            partial_ = DeviceBuf(ctx_, need * 4);
        }
    }
    // page tables of all slots behind `at`; longest: most tokens a sequence of the pass holds
    std::vector<uint32_t> page_table() const {
        std::vector<uint32_t> t((size_t)opt_.max_sequences * max_pages_, 0);
        for (uint32_t s = 0; s < opt_.max_sequences; ++s) std::copy(seqs_.pages(s).begin(), seqs_.pages(s).end(), t.begin() + (size_t)s * max_pages_);
        return t;
    }
    // Uploads a plan's tables and gives their device addresses.
    Rows upload(const PassPlan& plan, DeviceBuf& buf, uint32_t longest, const uint32_t** want) {
        Rows r;
        r.rows = plan.rows();
        r.latent_rows = plan.latent_rows;
        // portions whose attention runs head by head: their page lists, and blocks of queries, those that see most keys first
        uint32_t fewest_heads = 0xffffffffu, blocks = 0;
        for (const Layer& l : layers_) fewest_heads = std::min(fewest_heads, l.a.heads);
        for (const Portion& p : plan.portions) blocks += p.per_head ? (p.n + 127) / 128 : 0;
        r.job_rows = (uint64_t)blocks * fewest_heads >= kCus ? 128u : 64u;
        std::vector<uint32_t> list;
        struct Job { uint32_t row, n, first, keys; };
        std::vector<Job> jobs;
        for (const Portion& p : plan.portions) {
            if (!p.per_head) continue;
            const uint32_t first = (uint32_t)list.size(), len0 = p.length - p.n;
            list.insert(list.end(), seqs_.pages(p.slot).begin(), seqs_.pages(p.slot).begin() + seqs_.pages_for(p.length));
            for (uint32_t i = 0; i < p.n; i += r.job_rows) {
                const uint32_t n = std::min(r.job_rows, p.n - i);
                jobs.push_back({p.row + i, n, first, len0 + i + n});
            }
        }
        std::stable_sort(jobs.begin(), jobs.end(), [](const Job& a, const Job& b) { return a.keys > b.keys; });
        std::vector<uint32_t> job_words;
        for (const Job& j : jobs) job_words.insert(job_words.end(), {j.row, j.n, j.first, 0u});
        r.n_jobs = (uint32_t)jobs.size();
        r.n_pages = (uint32_t)list.size();
        std::vector<uint32_t> all;
        auto put = [&](const std::vector<uint32_t>& v) { const size_t at = all.size(); all.insert(all.end(), v.begin(), v.end()); return at; };
        const size_t tok = put(plan.tokens), prev = put(plan.prev), slot = put(plan.slot), pos = put(plan.pos), w = put(plan.want), table = put(page_table()),
                     jobs_at = put(job_words), list_at = put(list);
        std::vector<size_t> tiles_at;
        for (const TileSet& s : tile_sets_) {
            std::vector<uint32_t> t;
            Rows::Tiles d;
            make_tiles(s, plan.portions, t, d.m_tiles);
            d.n = (uint32_t)t.size() / 2;
            d.splits = choose_splits(opt_.act_dtype == M40LLM_ACT_F32 ? r.latent_rows * s.heads : d.n, longest);
            r.tiles.push_back(d);
            tiles_at.push_back(put(t));
        }
        if (buf.bytes() < all.size() * 4) buf = DeviceBuf(ctx_, all.size() * 4 + all.size());
        M40H_TRY(m40llm_memcpy_h2d(ctx_, buf.ptr(), all.data(), all.size() * 4));
        r.tokens = buf.u32(tok); r.prev = buf.u32(prev); r.slot = buf.u32(slot); r.pos = buf.u32(pos); r.page_table = buf.u32(table);
        r.jobs = buf.u32(jobs_at); r.page_list = buf.u32(list_at);
        for (size_t i = 0; i < tiles_at.size(); ++i) r.tiles[i].table = buf.u32(tiles_at[i]);
        if (want) *want = buf.u32(w);
        return r;
    }

    M40llmPackedGemm product(const void* a, uint32_t lda, const DeviceBuf& w, uint32_t n_tiles, uint32_t k_tiles, uint32_t rows, uint32_t epilogue) const {
        M40llmPackedGemm g{};
        g.act_dtype = opt_.act_dtype; g.epilogue = epilogue;
        g.a = a; g.lda = lda; g.w = w.ptr(); g.n_tiles = n_tiles; g.k_tiles = k_tiles;
        g.rows = rows; g.batches = 1;
        return g;
    }
    void launch(const M40llmPackedGemm& g) { M40H_TRY(m40llm_ext_packed_gemm_async(ctx_, &g, kStream)); }
    char* act(const DeviceBuf& b, size_t elements) const { return static_cast<char*>(b.ptr()) + elements * es_; }

    void enqueue_embedding(const Rows& r) {
        pending_ = 0;
        const BigramSpec b = spec_.bigram.value_or(BigramSpec{});
        M40H_TRY(m40llm_ext_embed_pairs_async(ctx_, embed_.ptr(), spec_.bigram ? bigram_.ptr() : nullptr, r.tokens, r.prev, r.rows, spec_.vocab,
                                              spec_.width, b.buckets, b.mul_prev, b.mul_cur, x_.ptr(), kStream));
        for (Rotation& t : rotations_)
            M40H_TRY(m40llm_ext_rotation_angles_async(ctx_, r.pos, r.rows, static_cast<const double*>(t.freq.ptr()), t.spec.dims / 2, t.half,
                                                      (float)t.spec.magnitude(), t.angles.ptr(), kStream));
    }
    void enqueue_layer(Layer& l, const Rows& r) {
        const LatentAttentionSpec& a = l.a;
        const Rotation& rot = rotations_[(size_t)l.rotation];
        DeviceBuf& cache = a.kv_from >= 0 ? layers_[(size_t)a.kv_from].cache : l.cache;
        M40H_TRY(m40llm_ext_layer_norm_rows_async(ctx_, x_.ptr(), planes_.ptr(), pending_, (uint64_t)r.rows * spec_.width, l.norm1.ptr(), nullptr,
                                                  r.rows, spec_.width, spec_.eps, h_.ptr(), d_pad_, opt_.act_dtype, kStream));
        pending_ = 0;
        const uint32_t ld_proj = l.plain_tiles * 16;
        {
            M40llmPackedGemm g = product(h_.ptr(), d_pad_, l.w_proj, l.proj_tiles, d_pad_ / 32, r.rows, M40LLM_PACKED_PROJECT);
            g.plain_tiles = l.plain_tiles;
            g.out_f32 = proj_.ptr(); g.ld_out = ld_proj;
            g.out_act = cat_.ptr(); g.ld_act = l.cat; g.act_col = l.o_pad;
            launch(g);
        }
        {
            M40llmLatentSplit s{};
            s.act_dtype = opt_.act_dtype; s.rows = r.rows;
            s.proj = proj_.ptr(); s.ld_proj = ld_proj;
            s.q_rank = a.q_rank; s.kv_offset = l.kv_offset; s.kv_rank = a.kv_rank; s.rot_offset = l.rot_offset; s.rot_dim = a.rot_dim;
            s.q_norm = l.q_norm.ptr(); s.kv_norm = l.kv_norm.ptr(); s.eps = spec_.eps;
            s.cq = cq_.ptr(); s.ld_cq = l.cq_pad;
            s.cache = a.kv_from < 0 ? cache.ptr() : nullptr;
            s.latent_pad = l.latent_pad; s.entry_width = l.entry_width; s.rot_half = rot.half;
            s.angles = rot.angles.ptr();
            s.row_slot = r.slot; s.row_pos = r.pos; s.page_table = r.page_table; s.max_pages = max_pages_;
            M40H_TRY(m40llm_ext_latent_split_append_async(ctx_, &s, kStream));
        }
        {
            M40llmPackedGemm g = product(cq_.ptr(), l.cq_pad, l.w_uq, a.heads * l.q_width / 16, l.cq_pad / 32, r.rows, M40LLM_PACKED_ROTATE);
            g.out_act = q_.ptr(); g.ld_act = (uint64_t)a.heads * l.q_width;
            g.head_width = l.q_width; g.rot_start = l.dim_pad; g.heads = a.heads; g.split_row = r.latent_rows; g.rot_half = rot.half;
            g.angles = rot.angles.ptr();
            g.rot_out = act(qa_, l.latent_pad); g.ld_rot = l.entry_width;
            launch(g);
        }
        if (r.latent_rows) enqueue_latent_attention(l, r, cache);
        if (r.n_jobs) enqueue_head_attention(l, r, cache);
        {
            M40llmPackedGemm g = product(cat_.ptr(), l.cat, l.w_out, round_up(spec_.width, 16) / 16, l.cat / 32, r.rows, M40LLM_PACKED_ADD);
            g.ld_out = spec_.width; g.cols = spec_.width;
            const uint32_t parts = r.in_place ? 1u : k_parts(g.n_tiles, g.k_tiles, r.rows);
            if (parts > 1u) {       // sums of parts of K: the next norm adds them to x
                g.epilogue = M40LLM_PACKED_STORE;
                g.k_parts = parts;
                g.out_f32 = planes_.ptr(); g.out_batch = (uint64_t)r.rows * spec_.width;
                pending_ = parts;
            } else {
                g.out_f32 = x_.ptr();
            }
            launch(g);
        }
    }
    // decoded tokens and short portions: rows before r.latent_rows
    void enqueue_latent_attention(Layer& l, const Rows& r, DeviceBuf& cache) {
        const LatentAttentionSpec& a = l.a;
        const uint32_t ld_proj = l.plain_tiles * 16;
        {
            M40llmPackedGemm g = product(q_.ptr(), a.heads * l.q_width, l.w_ukt, l.latent_pad / 16, l.dim_pad / 32, r.latent_rows, M40LLM_PACKED_STORE_ACT);
            g.batches = a.heads; g.a_batch = l.q_width; g.w_batch = (uint64_t)(l.latent_pad / 16) * (l.dim_pad / 32) * 512;
            g.out_act = qa_.ptr(); g.ld_act = (uint64_t)a.heads * l.entry_width; g.act_batch = l.entry_width; g.cols = l.latent_pad;
            launch(g);
        }
        {
            const Rows::Tiles& t = r.tiles[(size_t)l.tile_set];
            M40llmLatentAttention g{};
            g.act_dtype = opt_.act_dtype; g.heads = a.heads; g.kv_rank = a.kv_rank; g.latent_pad = l.latent_pad; g.entry_width = l.entry_width;
            g.scale = l.scale;
            g.queries = qa_.ptr(); g.cache = cache.ptr(); g.sink = l.sink.ptr();
            g.row_slot = r.slot; g.row_pos = r.pos; g.page_table = r.page_table; g.max_pages = max_pages_;
            g.tiles = t.table; g.n_tiles = t.n; g.m_tiles = t.m_tiles; g.splits = t.splits;
            g.first_query = 0; g.n_queries = r.latent_rows * a.heads;
            g.partial = partial_.ptr(); g.partial_floats = partial_.bytes() / 4;
            g.out = ol_.ptr();
            M40H_TRY(m40llm_ext_latent_attention_async(ctx_, &g, kStream));
        }
        {
            M40llmPackedGemm g = product(ol_.ptr(), a.heads * l.latent_pad, l.w_uv, l.vdim_tiles, l.latent_pad / 32, r.latent_rows, M40LLM_PACKED_GATED);
            g.batches = a.heads; g.a_batch = l.latent_pad; g.w_batch = (uint64_t)l.vdim_tiles * (l.latent_pad / 32) * 512;
            g.out_act = cat_.ptr(); g.ld_act = l.cat; g.act_batch = a.vdim; g.cols = a.vdim;
            g.gate = proj_.f32(l.gate_offset); g.ld_gate = ld_proj;
            launch(g);
        }
    }
    // long portions: rows from r.latent_rows on
    void enqueue_head_attention(Layer& l, const Rows& r, DeviceBuf& cache) {
        const LatentAttentionSpec& a = l.a;
        for (uint32_t kind : {M40LLM_PACKED_KEYS, M40LLM_PACKED_VALUES}) {
            const bool keys = kind == M40LLM_PACKED_KEYS;
            M40llmPackedGemm g = product(cache.ptr(), 0, keys ? l.w_uk : l.w_uv, keys ? a.heads * l.dim_pad / 16 : a.heads * l.vdim_tiles,
                                         l.latent_pad / 32, r.n_pages * kPage, kind);
            g.pages = r.page_list; g.page_k_tiles = l.entry_width / 32;
            g.out_act = keys ? keys_.ptr() : values_.ptr();
            launch(g);
        }
        M40llmHeadAttention h{};
        h.heads = a.heads; h.plain_tiles = l.dim_pad / 32; h.rot_tiles = l.rot_pad / 32; h.entry_tiles = l.entry_width / 32;
        h.vdim = a.vdim; h.v_tiles = l.vdim_tiles; h.scale = l.scale;
        h.queries = q_.ptr(); h.ld_queries = a.heads * l.q_width;
        h.keys = keys_.ptr(); h.values = values_.ptr(); h.cache = cache.ptr(); h.sink = l.sink.ptr();
        h.gate = proj_.f32(l.gate_offset); h.ld_gate = l.plain_tiles * 16;
        h.row_pos = r.pos; h.pages = r.page_list; h.jobs = r.jobs; h.n_jobs = r.n_jobs; h.job_rows = r.job_rows;
        h.out = cat_.ptr(); h.ld_out = l.cat;
        M40H_TRY(m40llm_ext_head_attention_async(ctx_, &h, kStream));
    }
    // Into how many parts the sum over the attention and feed-forward columns is cut where a launch would leave CUs idle.
    uint32_t k_parts(uint32_t n_tiles, uint32_t k_tiles, uint32_t rows) const {
        uint32_t groups;
        if (rows <= 64 || opt_.act_dtype == M40LLM_ACT_F32) groups = n_tiles * ((rows + 63) / 64);
        else groups = (rows + 127) / 128 * ((n_tiles + 7) / 8);
        uint32_t parts = 1;
        while (parts < kMaxParts && groups * parts * 2 <= kCus && k_tiles / (parts * 2) >= 32) parts *= 2;
        return (parts - 1) * ((k_tiles + parts - 1) / parts) < k_tiles ? parts : 1u;
    }
    // final norm and head of n of a pass's rows (row_index NULL = all of them)
    void enqueue_logits(const uint32_t* row_index, uint32_t n, uint32_t rows) {
        M40H_TRY(m40llm_ext_layer_norm_rows_async(ctx_, x_.ptr(), planes_.ptr(), pending_, (uint64_t)rows * spec_.width, final_norm_.ptr(), row_index, n,
                                                  spec_.width, spec_.eps, hn_.ptr(), d_pad_, opt_.act_dtype, kStream));
        M40llmPackedGemm g = product(hn_.ptr(), d_pad_, head_, round_up(spec_.vocab, 16) / 16, d_pad_ / 32, n, M40LLM_PACKED_STORE);
        g.out_f32 = logits_.ptr(); g.ld_out = spec_.vocab; g.cols = spec_.vocab;
        launch(g);
    }

    void run_pass(const PassPlan& plan, float* logits_out, const std::function<void(uint32_t, uint32_t, const float*)>& on_layer, const StepPicks* picks) {
        uint32_t longest = 0;
        for (const Portion& p : plan.portions)
            if (!p.per_head) longest = std::max(longest, p.length);
        M40H_TRY(m40llm_stream_synchronize(ctx_, kStream));           // the tables of the pass before may still be read
        const uint32_t* want = nullptr;
        Rows r = upload(plan, tables_, longest, &want);
        r.in_place = (bool)on_layer;
        ensure_scratch(r);
        enqueue_embedding(r);
        for (size_t i = 0; i < layers_.size(); ++i) {
            enqueue_layer(layers_[i], r);
            if (on_layer) {
                M40H_TRY(m40llm_stream_synchronize(ctx_, kStream));
                on_layer((uint32_t)i, r.rows, x_.f32());
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

    // Device-driven greedy steps: token, token before, position and step counter stay on the device.  Falls back to the host
    // sampler (same cache entries, rewritten) when a pick was a near tie.
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
            seqs_.grow(s, (uint64_t)kv_lens[i] + total);
            len0[i] = kv_lens[i];
            prev0[i] = seqs_.previous_token(s);
            plan.tokens.push_back(first_tokens[i]);
            plan.prev.push_back(prev0[i]);
            plan.slot.push_back(s);
            plan.pos.push_back(kv_lens[i]);
            plan.portions.push_back({i, 1, s, kv_lens[i] + 1, false});
            ++plan.latent_rows;
            longest = std::max(longest, kv_lens[i] + total);
        }
        M40H_TRY(m40llm_stream_synchronize(ctx_, kStream));
        drop_graph();
        Rows r = upload(plan, loop_tables_, longest, nullptr);
        ensure_scratch(r);
        loop_state_ = cleared(ctx_, 16);
        loop_ids_ = DeviceBuf(ctx_, (size_t)rows * total * 4);
        loop_gaps_ = DeviceBuf(ctx_, (size_t)rows * total * 4);
        auto enqueue = [&]() {
            enqueue_embedding(r);
            for (Layer& l : layers_) enqueue_layer(l, r);
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
    uint32_t es_;
    SequencePages seqs_;
    uint32_t max_pages_ = 0, d_pad_ = 0, logits_rows_ = 0, mode_ = 2;
    uint32_t pending_ = 0;             // planes whose sums x has not taken yet
    bool per_head_served_ = false;
    float tie_guard_ = DecodeModel::kGreedyTieGuard;
    bool timed_fallback_ = false;
    std::vector<Layer> layers_;
    std::vector<Rotation> rotations_;
    std::vector<TileSet> tile_sets_;
    DeviceBuf embed_, bigram_, final_norm_, head_, staging_;
    DeviceBuf keys_, values_;           // of the long portions' sequences, one layer at a time
    DeviceBuf x_, planes_, h_, proj_, cat_, cq_, q_, qa_, ol_, hn_, logits_, pick_parts_, partial_, tables_;
    DeviceBuf loop_tables_, loop_state_, loop_ids_, loop_gaps_;
    M40llmCudaGraphExec* graph_ = nullptr;
};

// A folder with config.json and model.safetensors.
inline std::unique_ptr<LayeredDecoder> open_model_folder(M40llmCudaContext* ctx, const std::string& dir, const LayeredOptions& opt) {
    DecoderSpec spec = read_decoder_spec(read_text_file(dir + "/config.json"));
    SafetensorsFile file(dir + "/model.safetensors");
    return std::make_unique<LayeredDecoder>(ctx, std::move(spec), file, opt);
}

}  // namespace m40host
