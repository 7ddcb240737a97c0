// Driver for test_layered_host.py: the host-side parts of layered decoders that need no device, one command a line on standard input,
// one JSON line out.
#include <iostream>
#include <sstream>

#include "../m40-llm_amd/host/decoder_spec.hpp"
#include "../m40-llm_amd/host/page_pool.hpp"
#include "../m40-llm_amd/host/safetensors.hpp"
#include "../m40-llm_amd/host/scheduler.hpp"

extern "C" {      // the device side of the tensor readers
int m40llm_memcpy_h2d(M40llmCudaContext*, void* dst, const void* src, size_t n) { std::memcpy(dst, src, n); return 0; }
int m40llm_ext_fill_random_bf16_async(M40llmCudaContext*, void*, uint64_t, uint64_t, float, uint32_t) { return 0; }
}

using namespace m40host;

static std::string quoted(const std::string& s) {
    std::string o = "\"";
    for (char c : s) o += c == '"' || c == '\\' ? std::string("\\") + c : c == '\n' ? std::string(" ") : std::string(1, c);
    return o + "\"";
}

static void rotation(const RotationSpec& r) {
    std::cout << ", \"rot_dims\": " << r.dims << ", \"magnitude\": " << r.magnitude() << ", \"freq\": [";
    const std::vector<double> f = r.frequencies();
    for (size_t k = 0; k < f.size(); ++k) std::cout << (k ? ", " : "") << f[k];
    std::cout << "]";
}

static void attention(const AttentionSpec& a) {
    std::cout << "\"sizes\": [" << a.heads << ", " << a.kv_heads << ", " << a.dim << ", " << a.vdim << "], \"scale\": " << a.scale << ", \"flags\": [" << a.biases << ", "
              << a.projection_norm << ", " << a.column_gate << ", " << a.share_values << "], \"scores\": [" << a.head_norm << ", " << a.distance_slopes << ", " << a.sink << ", " << a.cap
              << ", " << a.window << "]";
    if (a.rotation) rotation(*a.rotation);
}

static void spec(std::istream& in) {
    std::string path;
    in >> path;
    const DecoderSpec d = read_decoder_spec(read_text_file(path));
    std::cout.precision(17);
    std::cout << "{\"architecture\": " << quoted(d.architecture) << ", \"vocab\": " << d.vocab << ", \"width\": " << d.width << ", \"eps\": " << d.eps
              << ", \"bigram\": " << (d.bigram ? (int64_t)d.bigram->buckets : -1) << ", \"embedding_scale\": " << d.embedding_scale << ", \"residual_mult\": " << d.residual_mult << ", \"positions\": " << d.positions << ", \"streams\": " << d.streams
              << ", \"tied_head\": " << (d.tied_head ? "true" : "false") << ", \"around_zero\": " << (d.norm_around_zero ? "true" : "false") << ", \"logits\": [" << d.logit_scale << ", " << d.logit_cap << "], \"norm_scalar\": "
              << (d.norm_scalar ? "true" : "false") << ", \"layers\": [";
    for (size_t i = 0; i < d.layers.size(); ++i) {
        std::cout << (i ? ", " : "");
        const LayerSpec& l = d.layers[i];
        if (const auto* a = std::get_if<LatentAttentionSpec>(&l.mixer)) {
            std::cout << "{\"sizes\": [" << a->heads << ", " << a->dim << ", " << a->rot_dim << ", " << a->vdim << ", " << a->kv_rank << ", " << a->q_rank
                      << "], \"scale\": " << a->scale << ", \"kv_from\": " << a->kv_from ;
            rotation(a->rotation);
        } else if (const auto* a = std::get_if<DifferentialAttentionSpec>(&l.mixer)) {
            std::cout << "{\"sizes\": [" << a->heads << ", " << a->kv_heads << ", " << a->dim << ", " << a->vdim << ", " << a->taps << "], \"scale\": " << a->scale
                      << ", \"diff\": " << a->diff << ", \"kv_from\": " << a->kv_from;
        } else if (const auto* a = std::get_if<AttentionSpec>(&l.mixer)) {
            std::cout << "{";
            attention(*a);
        } else if (const auto* a = std::get_if<ParallelSpec>(&l.mixer)) {
            std::cout << "{\"left\": {";
            attention(a->left);
            std::cout << "}, \"right\": [" << a->right.heads << ", " << a->right.dim << ", " << a->right.vdim << ", " << a->right.gate_cap << "], \"factors\": ["
                      << a->left_scale << ", " << a->right_scale << "]";
        } else if (const auto* a = std::get_if<ChannelDeltaSpec>(&l.mixer)) {
            std::cout << "{\"sizes\": [" << a->heads << ", " << a->kv_heads << ", " << a->dim << ", " << a->vdim << ", " << a->taps << "]";
        } else if (const auto* a = std::get_if<TimeMixingSpec>(&l.mixer)) {
            std::cout << "{\"sizes\": [" << a->heads << ", " << a->dim << "]";
        } else if (const auto* a = std::get_if<StateSpaceSpec>(&l.mixer)) {
            std::cout << "{\"sizes\": [" << a->heads << ", " << a->groups << ", " << a->state << ", " << a->vdim << ", " << a->taps << ", " << a->norm_groups << "]";
        } else {
            const LightningSpec& n = std::get<LightningSpec>(l.mixer);
            std::cout << "{\"sizes\": [" << n.heads << ", " << n.dim << ", " << n.vdim << "], \"decay\": [";
            for (size_t k = 0; k < n.decay.size(); ++k) std::cout << (k ? ", " : "") << n.decay[k];
            std::cout << "]";
        }
        const auto* g = std::get_if<GatedMlpSpec>(&l.mlp);
        std::cout << ", \"ff\": " << (g ? g->ff : 0) << ", \"silu\": " << (g && g->activation == Activation::Silu ? "true" : "false");
        std::cout << ", \"tensors_of\": " << l.tensors_of;
        if (const auto* p = std::get_if<PolyMlpSpec>(&l.mlp)) std::cout << ", \"poly\": " << p->ff;
        if (const auto* e = std::get_if<ExpertMlpSpec>(&l.mlp))
            std::cout << ", \"experts\": [" << e->experts << ", " << e->identity << ", " << e->top << ", " << e->ff << "], \"groups\": [" << e->groups << ", " << e->keep << "], \"router_scale\": " << e->scale
                      << ", \"correction\": " << (e->correction ? "true" : "false") << ", \"sigmoid\": " << (e->score == RouterScore::Sigmoid ? "true" : "false")
                      << ", \"weight_input\": " << (e->weight_input ? "true" : "false") << ", \"limit\": [" << e->limit << ", " << e->alpha << "], \"activation\": " << (int)e->activation;
        std::cout << "}";
    }
    std::cout << "]}\n";
}

// pages <n_pages> <page> <slots> then words: g slot tokens | r slot tokens | a slot tokens last | f slot
static void pages(std::istream& in) {
    uint32_t n, page, slots;
    in >> n >> page >> slots;
    SequencePages p(n, page, slots);
    std::string op;
    std::cout << "[";
    bool first = true;
    while (in >> op) {
        uint32_t slot = 0, tokens = 0, last = 0;
        in >> slot;
        std::string result = "true";
        try {
            if (op == "g") { in >> tokens; p.grow(slot, tokens); }
            else if (op == "r") { in >> tokens; result = p.reserve(slot, tokens) ? "true" : "false"; }
            else if (op == "a") { in >> tokens >> last; p.advance(slot, tokens, last); }
            else if (op == "f") p.release(slot);
        } catch (const std::exception& e) {
            result = quoted(e.what());
        }
        std::cout << (first ? "" : ", ") << "{\"result\": " << result << ", \"free\": " << p.free_pages() << ", \"pages\": [";
        first = false;
        if (slot < slots)
            for (size_t i = 0; i < p.pages(slot).size(); ++i) std::cout << (i ? ", " : "") << p.pages(slot)[i];
        std::cout << "], \"length\": " << (slot < slots ? p.length(slot) : 0) << ", \"prev\": " << (slot < slots ? p.previous_token(slot) : 0) << "}";
    }
    std::cout << "]\n";
}

static void rows(std::istream& in) {
    std::string path, name;
    in >> path >> name;
    std::cout << SafetensorsFile(path).rows_of(name, 7) << "\n";
}

static void tensors(std::istream& in) {
    std::string path, name;
    in >> path >> name;
    std::vector<uint64_t> shape;
    for (uint64_t d; in >> d;) shape.push_back(d);
    SafetensorsFile f(path);
    const std::vector<float> v = f.read_f32(name, shape);
    std::cout << "[";
    for (size_t i = 0; i < v.size(); ++i) std::cout << (i ? ", " : "") << v[i];
    std::cout << "]\n";
}

// scheduler <step_tokens> <pool tokens> <slots> then p <prompt length> <max tokens> ... : every tick's items as [slot, start, len, want]
static void scheduler(std::istream& in) {
    uint32_t step_tokens, pool, slots;
    in >> step_tokens >> pool >> slots;
    constexpr uint32_t V = 50;
    SequencePages pages(pool / 4, 4, slots);
    std::ostringstream log;
    SchedulerEngine e;
    e.vocab = V;
    e.max_seq_len = pool;
    e.prefill = [](const std::vector<SchedulerPrefillItem>&, float*) { throw std::logic_error("not called where there is a step"); };
    e.decode = [](const std::vector<SchedulerDecodeItem>&, float*) { throw std::logic_error("not called where there is a step"); };
    e.reserve = [&](uint32_t s, uint64_t n) { return pages.reserve(s, n); };
    e.release = [&](uint32_t s) { pages.release(s); };
    e.step_tokens = step_tokens;
    bool first = true;
    e.step = [&](const std::vector<SchedulerStepItem>& items, const uint8_t* greedy, float* out, uint32_t* picks, uint8_t* picked) {
        log << (first ? "" : ", ") << "[";
        first = false;
        size_t row = 0;
        for (size_t i = 0; i < items.size(); ++i) {
            const SchedulerStepItem& it = items[i];
            if (pages.length(it.sequence_id) != it.start) throw std::logic_error("wrong start");
            pages.grow(it.sequence_id, it.start + it.len);
            pages.advance(it.sequence_id, it.len, it.tokens[it.len - 1]);
            log << (i ? ", " : "") << "[" << it.sequence_id << ", " << it.start << ", " << it.len << ", " << (it.want ? 1 : 0) << "]";
            if (!it.want) continue;
            const uint32_t next = (it.tokens[it.len - 1] + 1) % V;      // the next number, every other time as a pick
            picked[row] = greedy[row] && (it.start & 1);
            picks[row] = next;
            for (uint32_t v = 0; v < V; ++v) out[row * V + v] = v == (picked[row] ? 0 : next) ? 1.0f : 0.0f;
            ++row;
        }
        log << "]";
    };
    DecodeScheduler s(std::move(e), slots);
    std::vector<uint64_t> ids;
    std::string op;
    std::vector<std::pair<uint32_t, uint32_t>> todo;
    while (in >> op) {
        uint32_t n, m;
        in >> n >> m;
        todo.push_back({n, m});
    }
    SamplerConfig greedy;
    greedy.top_k = 1;
    size_t next = 0;
    for (int t = 0; t < 1000 && (next < todo.size() || s.active()); ++t) {
        while (next < todo.size() && s.available_slots()) {
            std::vector<uint32_t> prompt;
            for (uint32_t i = 0; i < todo[next].first; ++i) prompt.push_back((uint32_t)(10 * next + i) % V);
            ids.push_back(s.submit(prompt.data(), prompt.size(), todo[next].second, {}, greedy));
            ++next;
        }
        s.tick();
    }
    std::cout << "{\"ticks\": [" << log.str() << "], \"free\": " << pages.free_pages() << ", \"requests\": [";
    for (size_t i = 0; i < ids.size(); ++i) {
        std::cout << (i ? ", " : "") << "{\"state\": " << (int)s.state(ids[i]) << ", \"error\": " << quoted(s.error_of(ids[i])) << ", \"ids\": [";
        const auto g = s.generated(ids[i]);
        for (size_t k = 0; k < g.size(); ++k) std::cout << (k ? ", " : "") << g[k];
        std::cout << "]}";
    }
    std::cout << "]}\n";
}

int main() {
    std::string line;
    while (std::getline(std::cin, line)) {
        std::istringstream in(line);
        std::string what;
        in >> what;
        try {
            if (what == "spec") spec(in);
            else if (what == "pages") pages(in);
            else if (what == "tensors") tensors(in);
            else if (what == "rows") rows(in);
            else if (what == "scheduler") scheduler(in);
        } catch (const std::exception& e) {
            std::cout << "{\"error\": " << quoted(e.what()) << "}\n";
        }
        std::cout.flush();
    }
    return 0;
}
