// A parallel block with latent attention.  Launches (all on the decode stream):
//   layer norm                      h = norm(x)
//   packed product, PROJECT         [q latent | kv latent | rotated key | gate logits] -> f32, activation(gate) * up -> bf16
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

#include "layer_runtime.hpp"

namespace m40host {

// Tiles of query rows (row, head) for the rows of single tokens and short portions.
struct LatentTiles : PassTable {
    LatentTiles(uint32_t act, uint32_t h, uint32_t most, uint32_t pad) : act_dtype(act), heads(h), max_m_tiles(most), latent_pad(pad) {}
    bool same(uint32_t, uint32_t h, uint32_t most, uint32_t pad) const { return heads == h && max_m_tiles == most && latent_pad == pad; }
    std::vector<uint32_t> build(const PassPlan& plan, const SequencePages&, uint32_t longest) override {
        uint32_t most = 0;
        for (const Portion& p : plan.portions)
            if (!p.is_long) most = std::max(most, p.n * heads);
        m_tiles = std::min(most <= 16 ? 1u : most <= 32 ? 2u : 4u, max_m_tiles);
        const uint32_t size = 16 * m_tiles;
        std::vector<uint32_t> t;
        for (const Portion& p : plan.portions)
            for (uint32_t i = 0; !p.is_long && i < p.n * heads; i += size) t.insert(t.end(), {p.row * heads + i, std::min(size, p.n * heads - i)});
        n = (uint32_t)t.size() / 2;
        const uint32_t pages = (longest + LayerRuntime::kPage - 1) / LayerRuntime::kPage, work = act_dtype == M40LLM_ACT_F32 ? plan.short_rows * heads : n;
        splits = std::max(1u, std::min(pages, 256u / std::max(work, 1u)));
        return t;
    }
    uint64_t partial_floats(const Rows& r) const override { return m40llm_ext_latent_attention_partial_floats(r.short_rows * heads, latent_pad, splits); }
    uint32_t act_dtype, heads, max_m_tiles, latent_pad, n = 0, m_tiles = 1, splits = 1;
};

// Long portions: blocks of queries, those that see most keys first, and the portions' page lists.
struct LatentJobs : PassTable {
    bool same() const { return true; }
    uint32_t fewest_heads = 0xffffffffu, n_jobs = 0, job_rows = 128, n_pages = 0;
    const uint32_t* list() const { return at + 4 * n_jobs; }
    std::vector<uint32_t> build(const PassPlan& plan, const SequencePages& pages, uint32_t) override {
        uint32_t blocks = 0;
        for (const Portion& p : plan.portions) blocks += p.is_long ? (p.n + 127) / 128 : 0;
        job_rows = (uint64_t)blocks * fewest_heads >= LayerRuntime::kCus ? 128u : 64u;
        std::vector<uint32_t> list;
        struct Job { uint32_t row, n, first, keys; };
        std::vector<Job> jobs;
        for (const Portion& p : plan.portions) {
            if (!p.is_long) continue;
            const uint32_t first = (uint32_t)list.size(), len0 = p.length - p.n;
            list.insert(list.end(), pages.pages(p.slot).begin(), pages.pages(p.slot).begin() + pages.pages_for(p.length));
            for (uint32_t i = 0; i < p.n; i += job_rows) {
                const uint32_t n = std::min(job_rows, p.n - i);
                jobs.push_back({p.row + i, n, first, len0 + i + n});
            }
        }
        std::stable_sort(jobs.begin(), jobs.end(), [](const Job& a, const Job& b) { return a.keys > b.keys; });
        std::vector<uint32_t> t;
        for (const Job& j : jobs) t.insert(t.end(), {j.row, j.n, j.first, 0u});
        n_jobs = (uint32_t)jobs.size();
        n_pages = (uint32_t)list.size();
        t.insert(t.end(), list.begin(), list.end());
        return t;
    }
};

// buffers all latent layers of a decoder share
struct LatentShared {
    Scratch cq, q, qa, ol;
    DeviceBuf keys, values;               // of the long portions' sequences, one layer at a time
    bool per_head_served = true;          // every layer's head sizes are served by the head attention
};

class LatentLayer : public DecoderLayer {
public:
    LatentLayer(LayerRuntime& rt, std::shared_ptr<LatentShared> shared, TensorSource& t, uint32_t index, const LayerSpec& s, LatentLayer* source)
        : rt_(rt), sh_(std::move(shared)), a_(std::get<LatentAttentionSpec>(s.mixer)), source_(source), jobs_(rt.table<LatentJobs>()) {
        const LatentAttentionSpec& a = a_;
        const GatedMlpSpec* mlp = std::get_if<GatedMlpSpec>(&s.mlp);
        ff_ = mlp ? mlp->ff : 0;
        activation_ = mlp && mlp->activation == Activation::Silu ? M40LLM_SILU : M40LLM_GELU_TANH;
        const bool own = !source;
        dim_pad_ = round_up(a.dim, 32); rot_pad_ = round_up(a.rot_dim, 32); q_width_ = dim_pad_ + rot_pad_;
        latent_pad_ = round_up(a.kv_rank, 32); entry_width_ = latent_pad_ + rot_pad_;
        cq_pad_ = round_up(a.q_rank, 32);
        kv_offset_ = round_up(a.q_rank, 16);
        rot_offset_ = kv_offset_ + (own ? round_up(a.kv_rank, 16) : 0);
        gate_offset_ = rot_offset_ + (own ? round_up(a.rot_dim, 16) : 0);
        plain_tiles_ = round_up(gate_offset_ + round_up(a.heads, 16), 32) / 16;
        proj_tiles_ = plain_tiles_ + 2 * (round_up(ff_, 16) / 16);
        o_pad_ = round_up(a.heads * a.vdim, 32);
        cat_ = o_pad_ + round_up(ff_, 32);
        vdim_tiles_ = round_up(a.vdim, 16) / 16;
        const uint32_t max_m = m40llm_ext_latent_attention_max_m_tiles(rt.opt.act_dtype, a.kv_rank, entry_width_);
        if (max_m == 0) throw std::invalid_argument("layer " + std::to_string(index) + ": kv_rank + rot_dim beyond what the attention kernels serve");
        rot_ = &rt.table<RotationAngles>(&rt, a.rotation, rot_pad_ / 2);
        tiles_ = &rt.table<LatentTiles>(rt.opt.act_dtype, a.heads, max_m, latent_pad_);
        jobs_.fewest_heads = std::min(jobs_.fewest_heads, a.heads);
        load(t, index, own);
        rt.proj.want(rt.f32_bytes((size_t)plain_tiles_ * 16));
        rt.cat.want(rt.act_bytes(cat_));
        sh_->cq.want(rt.act_bytes(cq_pad_));
        sh_->q.want(rt.act_bytes((size_t)a.heads * q_width_));
        sh_->qa.want(rt.act_bytes((size_t)a.heads * entry_width_));
        sh_->ol.want(rt.act_bytes((size_t)a.heads * latent_pad_));
        rt.want_planes(cat_ / 32, false);
    }

    // The latent form's kernel reaches half the rate of the head form's.
    bool portion_cost(uint32_t n, uint32_t len, double& as_tokens, double& as_long) const override {
        if (!sh_->per_head_served) return false;
        const double keys = (double)len + n, seen = (double)n * (len + n / 2.0);
        as_tokens += 2.0 * seen * a_.heads * (entry_width_ + latent_pad_) + (double)n * a_.heads * latent_pad_ * (dim_pad_ + a_.vdim);
        as_long += seen * a_.heads * (q_width_ + a_.vdim) + keys * a_.heads * latent_pad_ * (dim_pad_ + a_.vdim);
        return true;
    }
    void prepare(const Rows&) override {
        const uint64_t keys = (uint64_t)jobs_.n_pages * LayerRuntime::kPage * a_.heads * dim_pad_ * 2;
        const uint64_t values = (uint64_t)jobs_.n_pages * LayerRuntime::kPage * a_.heads * vdim_tiles_ * 16 * 2;
        if (keys > sh_->keys.bytes() || values > sh_->values.bytes()) {
            M40H_TRY(m40llm_stream_synchronize(rt_.ctx, rt_.kStream));
            sh_->keys = DeviceBuf(rt_.ctx, std::max<uint64_t>(keys, sh_->keys.bytes()));
            sh_->values = DeviceBuf(rt_.ctx, std::max<uint64_t>(values, sh_->values.bytes()));
        }
    }

    void enqueue(const Rows& r) override {
        const LatentAttentionSpec& a = a_;
        DeviceBuf& cache = source_ ? source_->cache_ : cache_;
        M40H_TRY(m40llm_ext_layer_norm_rows_async(rt_.ctx, rt_.x.ptr(), rt_.planes.ptr(), rt_.pending, (uint64_t)r.rows * rt_.spec.width, norm1_.ptr(), nullptr,
                                                  r.rows, rt_.spec.width, rt_.spec.eps, rt_.h.ptr(), rt_.d_pad, rt_.opt.act_dtype, rt_.kStream));
        rt_.pending = 0;
        const uint32_t ld_proj = plain_tiles_ * 16;
        {
            M40llmPackedGemm g = rt_.product(rt_.h.ptr(), rt_.d_pad, w_proj_, proj_tiles_, rt_.d_pad / 32, r.rows, M40LLM_PACKED_PROJECT);
            g.plain_tiles = plain_tiles_; g.activation = activation_;
            g.out_f32 = rt_.proj.ptr(); g.ld_out = ld_proj;
            g.out_act = rt_.cat.ptr(); g.ld_act = cat_; g.act_col = o_pad_;
            rt_.launch(g);
        }
        {
            M40llmLatentSplit s{};
            s.act_dtype = rt_.opt.act_dtype; s.rows = r.rows;
            s.proj = rt_.proj.ptr(); s.ld_proj = ld_proj;
            s.q_rank = a.q_rank; s.kv_offset = kv_offset_; s.kv_rank = a.kv_rank; s.rot_offset = rot_offset_; s.rot_dim = a.rot_dim;
            s.q_norm = q_norm_.ptr(); s.kv_norm = kv_norm_.ptr(); s.eps = rt_.spec.eps;
            s.cq = sh_->cq.ptr(); s.ld_cq = cq_pad_;
            s.cache = source_ ? nullptr : cache.ptr();
            s.latent_pad = latent_pad_; s.entry_width = entry_width_; s.rot_half = rot_->half;
            s.angles = rot_->angles.ptr();
            s.row_slot = r.slot; s.row_pos = r.pos; s.page_table = r.page_table; s.max_pages = rt_.max_pages;
            M40H_TRY(m40llm_ext_latent_split_append_async(rt_.ctx, &s, rt_.kStream));
        }
        {
            M40llmPackedGemm g = rt_.product(sh_->cq.ptr(), cq_pad_, w_uq_, a.heads * q_width_ / 16, cq_pad_ / 32, r.rows, M40LLM_PACKED_ROTATE);
            g.out_act = sh_->q.ptr(); g.ld_act = (uint64_t)a.heads * q_width_;
            g.head_width = q_width_; g.rot_start = dim_pad_; g.heads = a.heads; g.split_row = r.short_rows; g.rot_half = rot_->half;
            g.angles = rot_->angles.ptr();
            g.rot_out = rt_.act(sh_->qa.ptr(), latent_pad_); g.ld_rot = entry_width_;
            rt_.launch(g);
        }
        if (r.short_rows) latent_attention(r, cache);
        if (jobs_.n_jobs) head_attention(r, cache);
        {
            M40llmPackedGemm g = rt_.product(rt_.cat.ptr(), cat_, w_out_, round_up(rt_.spec.width, 16) / 16, cat_ / 32, r.rows, M40LLM_PACKED_ADD);
            g.ld_out = rt_.spec.width; g.cols = rt_.spec.width;
            if (!r.in_place && rt_.k_parts(g.n_tiles, g.k_tiles, r.rows) > 1u) {       // the next norm adds the parts' sums to x
                rt_.pending = rt_.into_planes(g, r.rows);
            } else {
                g.out_f32 = rt_.x.ptr();
                rt_.launch(g);
            }
        }
    }

private:
    void load(TensorSource& t, uint32_t index, bool own) {
        const LatentAttentionSpec& a = a_;
        const uint32_t D = rt_.spec.width, d_tiles = rt_.d_pad / 32;
        const std::string p = "l" + std::to_string(index) + ".", x = p + "mix.";
        norm1_ = rt_.upload_f32(t.read_f32(p + "norm1", {D}));
        q_norm_ = rt_.upload_f32(t.read_f32(x + "dq.norm", {a.q_rank}));
        sink_ = rt_.upload_f32(t.read_f32(x + "sink", {a.heads}));
        w_proj_ = rt_.packed(proj_tiles_, d_tiles);
        rt_.pack(t, x + "dq", a.q_rank, D, w_proj_.ptr(), d_tiles, 0);
        if (own) {
            kv_norm_ = rt_.upload_f32(t.read_f32(x + "dkv.norm", {a.kv_rank}));
            const void* src = rt_.stage(t, x + "dkv", {a.kv_rank + a.rot_dim, D});
            rt_.pack_rows(src, 0, a.kv_rank, D, w_proj_.ptr(), d_tiles, kv_offset_ / 16);
            rt_.pack_rows(src, a.kv_rank, a.rot_dim, D, w_proj_.ptr(), d_tiles, rot_offset_ / 16);
        }
        rt_.pack(t, x + "g", a.heads, D, w_proj_.ptr(), d_tiles, gate_offset_ / 16);
        if (ff_) {
            rt_.pack(t, p + "mlp.gate", ff_, D, w_proj_.ptr(), d_tiles, plain_tiles_, 0, 2);
            rt_.pack(t, p + "mlp.up", ff_, D, w_proj_.ptr(), d_tiles, plain_tiles_ + 1, 0, 2);
        }
        {
            const uint32_t kt = cq_pad_ / 32;
            w_uq_ = rt_.packed(a.heads * q_width_ / 16, kt);
            const void* src = rt_.stage(t, x + "uq", {(uint64_t)a.heads * (a.dim + a.rot_dim), a.q_rank});
            rt_.pack_heads(src, a.heads, a.dim + a.rot_dim, 0, a.dim, a.q_rank, w_uq_.ptr(), kt, q_width_, 0);
            rt_.pack_heads(src, a.heads, a.dim + a.rot_dim, a.dim, a.rot_dim, a.q_rank, w_uq_.ptr(), kt, q_width_, dim_pad_);
        }
        {   // W_uk [heads * dim][kv_rank] as one [kv_rank][dim] matrix a head
            w_ukt_ = rt_.packed(a.heads * latent_pad_ / 16, dim_pad_ / 32);
            const void* src = rt_.stage(t, x + "uk", {(uint64_t)a.heads * a.dim, a.kv_rank});
            M40llmPackPlan q{};
            q.n_blocks = a.heads; q.n = a.kv_rank; q.n_block_pad = latent_pad_;
            q.k_blocks = 1; q.k = a.dim; q.k_block_pad = a.dim;
            q.sn_block = (uint64_t)a.dim * a.kv_rank; q.sn = 1; q.sk = a.kv_rank;
            q.k_tiles = dim_pad_ / 32; q.tile_stride = 1;
            M40H_TRY(m40llm_ext_pack_tiles_async(rt_.ctx, src, w_ukt_.ptr(), &q, rt_.kStream));
            if (sh_->per_head_served) {
                w_uk_ = rt_.packed(a.heads * dim_pad_ / 16, latent_pad_ / 32);
                rt_.pack_heads(src, a.heads, a.dim, 0, a.dim, a.kv_rank, w_uk_.ptr(), latent_pad_ / 32, dim_pad_, 0);
            }
        }
        {
            const uint32_t kt = latent_pad_ / 32;
            w_uv_ = rt_.packed(a.heads * vdim_tiles_, kt);
            const void* src = rt_.stage(t, x + "uv", {(uint64_t)a.heads * a.vdim, a.kv_rank});
            rt_.pack_heads(src, a.heads, a.vdim, 0, a.vdim, a.kv_rank, w_uv_.ptr(), kt, vdim_tiles_ * 16, 0);
        }
        w_out_ = rt_.packed(round_up(D, 16) / 16, cat_ / 32);
        rt_.pack(t, x + "o", D, a.heads * a.vdim, w_out_.ptr(), cat_ / 32, 0, 0);
        if (ff_) rt_.pack(t, p + "mlp.down", D, ff_, w_out_.ptr(), cat_ / 32, 0, o_pad_);
        if (own) cache_ = rt_.cleared((size_t)rt_.max_pages * LayerRuntime::kPage * entry_width_ * rt_.es);
    }
    // decoded tokens and short portions: rows before r.short_rows
    void latent_attention(const Rows& r, DeviceBuf& cache) {
        const LatentAttentionSpec& a = a_;
        const uint32_t ld_proj = plain_tiles_ * 16;
        {
            M40llmPackedGemm g = rt_.product(sh_->q.ptr(), a.heads * q_width_, w_ukt_, latent_pad_ / 16, dim_pad_ / 32, r.short_rows, M40LLM_PACKED_STORE_ACT);
            g.batches = a.heads; g.a_batch = q_width_; g.w_batch = (uint64_t)(latent_pad_ / 16) * (dim_pad_ / 32) * 512;
            g.out_act = sh_->qa.ptr(); g.ld_act = (uint64_t)a.heads * entry_width_; g.act_batch = entry_width_; g.cols = latent_pad_;
            rt_.launch(g);
        }
        {
            M40llmLatentAttention g{};
            g.act_dtype = rt_.opt.act_dtype; g.heads = a.heads; g.kv_rank = a.kv_rank; g.latent_pad = latent_pad_; g.entry_width = entry_width_;
            g.scale = a.scale;
            g.queries = sh_->qa.ptr(); g.cache = cache.ptr(); g.sink = sink_.ptr();
            g.row_slot = r.slot; g.row_pos = r.pos; g.page_table = r.page_table; g.max_pages = rt_.max_pages;
            g.tiles = tiles_->at; g.n_tiles = tiles_->n; g.m_tiles = tiles_->m_tiles; g.splits = tiles_->splits;
            g.first_query = 0; g.n_queries = r.short_rows * a.heads;
            g.partial = rt_.partial.ptr(); g.partial_floats = rt_.partial.bytes() / 4;
            g.out = sh_->ol.ptr();
            M40H_TRY(m40llm_ext_latent_attention_async(rt_.ctx, &g, rt_.kStream));
        }
        {
            M40llmPackedGemm g = rt_.product(sh_->ol.ptr(), a.heads * latent_pad_, w_uv_, vdim_tiles_, latent_pad_ / 32, r.short_rows, M40LLM_PACKED_GATED);
            g.batches = a.heads; g.a_batch = latent_pad_; g.w_batch = (uint64_t)vdim_tiles_ * (latent_pad_ / 32) * 512;
            g.out_act = rt_.cat.ptr(); g.ld_act = cat_; g.act_batch = a.vdim; g.cols = a.vdim;
            g.gate = rt_.proj.f32(gate_offset_); g.ld_gate = ld_proj;
            rt_.launch(g);
        }
    }
    // long portions: rows from r.short_rows on
    void head_attention(const Rows& r, DeviceBuf& cache) {
        const LatentAttentionSpec& a = a_;
        for (uint32_t kind : {M40LLM_PACKED_KEYS, M40LLM_PACKED_VALUES}) {
            const bool keys = kind == M40LLM_PACKED_KEYS;
            M40llmPackedGemm g = rt_.product(cache.ptr(), 0, keys ? w_uk_ : w_uv_, keys ? a.heads * dim_pad_ / 16 : a.heads * vdim_tiles_, latent_pad_ / 32,
                                             jobs_.n_pages * LayerRuntime::kPage, kind);
            g.pages = jobs_.list(); g.page_k_tiles = entry_width_ / 32;
            g.out_act = keys ? sh_->keys.ptr() : sh_->values.ptr();
            rt_.launch(g);
        }
        M40llmHeadAttention h{};
        h.heads = a.heads; h.plain_tiles = dim_pad_ / 32; h.rot_tiles = rot_pad_ / 32; h.entry_tiles = entry_width_ / 32;
        h.vdim = a.vdim; h.v_tiles = vdim_tiles_; h.scale = a.scale;
        h.queries = sh_->q.ptr(); h.ld_queries = a.heads * q_width_;
        h.keys = sh_->keys.ptr(); h.values = sh_->values.ptr(); h.cache = cache.ptr(); h.sink = sink_.ptr();
        h.gate = rt_.proj.f32(gate_offset_); h.ld_gate = plain_tiles_ * 16;
        h.row_pos = r.pos; h.pages = jobs_.list(); h.jobs = jobs_.at; h.n_jobs = jobs_.n_jobs; h.job_rows = jobs_.job_rows;
        h.out = rt_.cat.ptr(); h.ld_out = cat_;
        M40H_TRY(m40llm_ext_head_attention_async(rt_.ctx, &h, rt_.kStream));
    }

    LayerRuntime& rt_;
    std::shared_ptr<LatentShared> sh_;
    LatentAttentionSpec a_;
    LatentLayer* source_;                 // whose cache it reads (null = its own)
    LatentJobs& jobs_;
    RotationAngles* rot_;
    LatentTiles* tiles_;
    uint32_t ff_, activation_;            // ff 0 = no feed-forward
    uint32_t dim_pad_, rot_pad_, q_width_;   // a head's query: [dim_pad | rot_pad]
    uint32_t latent_pad_, entry_width_, cq_pad_;
    uint32_t plain_tiles_, proj_tiles_, kv_offset_, rot_offset_, gate_offset_;
    uint32_t o_pad_, cat_;                // [attention | feed-forward] columns
    uint32_t vdim_tiles_;
    DeviceBuf norm1_, w_proj_, q_norm_, kv_norm_, w_uq_, w_ukt_, w_uk_, w_uv_, sink_, w_out_, cache_;
};

}  // namespace m40host
