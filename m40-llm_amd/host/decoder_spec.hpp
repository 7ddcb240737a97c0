// What a layered decoder is made of, and the registry that reads it from a model folder's config.json: "architecture" names the
// design, the design's reader turns the rest into a DecoderSpec.  Mechanisms take their constants from here, so that another
// design can combine them differently.
#pragma once

#include <algorithm>
#include <cmath>
#include <cstdint>
#include <fstream>
#include <functional>
#include <map>
#include <optional>
#include <sstream>
#include <string>
#include <variant>
#include <vector>

#include "json.hpp"

namespace m40host {

// Rotary positions on the first `dims` dimensions, pairs (2 i, 2 i + 1), frequencies base^(-2 i / dims); with YaRN scaling the low
// frequencies are divided by `factor`, a ramp between the dimensions that turn `fast` and `slow` times within `original`
// positions joins the two, and cos and sin carry a magnitude.
struct RotationSpec {
    uint32_t dims = 0;
    double base = 10000.0;
    bool scaled = false;
    double factor = 1.0, original = 0.0, fast = 0.0, slow = 0.0;
    bool operator==(const RotationSpec& o) const {
        return dims == o.dims && base == o.base && scaled == o.scaled && factor == o.factor && original == o.original && fast == o.fast &&
               slow == o.slow;
    }
    std::vector<double> frequencies() const {
        std::vector<double> f(dims / 2);
        for (uint32_t i = 0; i < dims / 2; ++i) f[i] = std::pow(base, -2.0 * i / dims);
        if (!scaled) return f;
        auto dim_of = [&](double turns) { return dims * std::log(original / (2.0 * M_PI * turns)) / (2.0 * std::log(base)); };
        const double lo = std::max(std::floor(dim_of(fast)), 0.0), hi = std::min(std::ceil(dim_of(slow)), (double)dims - 1.0);
        for (uint32_t i = 0; i < dims / 2; ++i) {
            const double ramp = std::min(std::max((i - lo) / std::max(hi - lo, 0.001), 0.0), 1.0);
            f[i] = f[i] / factor * ramp + f[i] * (1.0 - ramp);
        }
        return f;
    }
    double magnitude() const { return scaled ? 0.1 * std::log(factor) + 1.0 : 1.0; }
};

// Queries through a latent of q_rank; keys and values from a latent of kv_rank, cached with one rotated key part of rot_dim for
// all heads; a sink per head in the softmax denominator; a sigmoid gate per head.  kv_from >= 0: reads that layer's cache.
struct LatentAttentionSpec {
    uint32_t heads = 0, dim = 0, rot_dim = 0, vdim = 0, kv_rank = 0, q_rank = 0;
    float scale = 0.0f;
    int kv_from = -1;
    RotationSpec rotation;
};

// Every head two softmax maps over the same values, the second's result taken off the first's; queries, keys and values pass a causal
// convolution of `taps` taps (0 = none) and per-map norms; a sigmoid gate per head.  kv_from >= 0: reads that layer's cache.
struct DifferentialAttentionSpec {
    uint32_t heads = 0, kv_heads = 0, dim = 0, vdim = 0, taps = 0;
    float scale = 0.0f;
    double diff = 0.0;             // added to the second map's weight; the result is scaled by one less it
    int kv_from = -1;
};

// Linear attention whose state decays by one factor a head; norm over all heads and a sigmoid gate per column before the output product.
struct LightningSpec {
    uint32_t heads = 0, dim = 0, vdim = 0;
    std::vector<double> decay;
};

// Softmax attention.  Optional: biases on the projections, RMS norm over all query and over all key columns, rotation, a sigmoid gate per
// column; values mixed with those of the first layer that shares its own (share_values); RMS norm of every query and key head without a weight;
// scores held within +-cap by a tanh; less a slope times the distance of key and query, 2^(-8 (h + 1) / heads) for head h; a window of the newest
// tokens; a sink per head in the denominator.
struct AttentionSpec {
    uint32_t heads = 0, kv_heads = 0, dim = 0, vdim = 0;
    float scale = 0.0f;
    bool biases = false, projection_norm = false, column_gate = false, share_values = false, head_norm = false, distance_slopes = false, sink = false;
    float cap = 0.0f;              // 0 = none
    uint32_t window = 0;           // 0 = all
    std::optional<RotationSpec> rotation;
};

// A matrix state with exponential gates whose logits are capped; norm per head, weights per column, a sigmoid gate per column.
struct MatrixMemorySpec {
    uint32_t heads = 0, dim = 0, vdim = 0;
    float gate_cap = 0.0f;
};

// Attention and a matrix memory that read the same input; their outputs times a factor each.
struct ParallelSpec {
    AttentionSpec left;
    MatrixMemorySpec right;
    float left_scale = 1.0f, right_scale = 1.0f;
};

// Delta rule with one decay per head and key channel; queries, keys and values behind a short convolution and silu; decays and output gates from
// low-rank products whose rank the tensors give.
struct ChannelDeltaSpec {
    uint32_t heads = 0, kv_heads = 0, dim = 0, vdim = 0, taps = 0;
};

// Time mixing (RWKV): receptance, keys, values, gates and decays each from their own mix of a token with the one before; one decay per head and key
// channel, from a low-rank product whose rank the tensors give; a bonus for the current token.
struct TimeMixingSpec {
    uint32_t heads = 0, dim = 0;
};

// State space layer (Mamba-2): values, keys and queries (heads of a group share the latter two) behind a short convolution; decay and input weight from a
// step size per token and head; a direct part; a gate, then an RMS norm over each of norm_groups parts.
struct StateSpaceSpec {
    uint32_t heads = 0, groups = 0, state = 0, vdim = 0, taps = 0, norm_groups = 0;
};

typedef std::variant<LatentAttentionSpec, DifferentialAttentionSpec, LightningSpec, AttentionSpec, ParallelSpec, ChannelDeltaSpec, TimeMixingSpec, StateSpaceSpec> MixerSpec;

enum class Activation { GeluTanh, Silu, LimitedGate };
enum class RouterScore { Softmax, Sigmoid };
enum class NormKind { Layer, Rms };

struct GatedMlpSpec {          // down(activation(gate h) * (up h))
    uint32_t ff = 0;
    Activation activation = Activation::GeluTanh;
};

struct PolyMlpSpec {           // down(p(up h)), p a polynomial whose powers are each divided by their root mean square
    uint32_t ff = 0;
};

// Of `experts` gated feed-forwards and `identity` experts that return their input, each token takes `top` by score (+ correction)
// and adds up their outputs times scale times their scores, or (weight_input) their outputs for its input times scale times their scores.  groups > 1: experts form groups of neighbours, and only those of the `keep` groups with
// the best expert can be taken.
struct ExpertMlpSpec {
    uint32_t experts = 0, identity = 0, top = 0, ff = 0, groups = 1, keep = 1;
    float scale = 1.0f;
    bool correction = true, weight_input = false;
    RouterScore score = RouterScore::Softmax;
    Activation activation = Activation::Silu;
    float limit = 0.0f, alpha = 1.0f;        // LimitedGate
};

typedef std::variant<std::monostate, GatedMlpSpec, ExpertMlpSpec, PolyMlpSpec> MlpSpec;

struct BigramSpec {            // a second embedding looked up by (token before, token)
    uint32_t buckets = 0, mul_prev = 0, mul_cur = 0;
};

struct LayerSpec {
    MixerSpec mixer;
    MlpSpec mlp;
    int tensors_of = -1;               // the layer whose tensors it uses (-1 = its own)
};

enum class BlockKind {
    Parallel,       // one norm whose output both sublayers read: x += mixer(norm(x)) + mlp(norm(x))
    OutputNorm,     // x += m * norm1(mixer(x)), then x += m * norm2(mlp(x))
    PreNorm,        // x += mixer(norm1(x)), then x += mlp(norm2(x))
    Streams,        // several streams: u = in . x, y = mixer(norm1(u)), x_t = sum_s mix[s][t] x_s + m * out[t] * y; the same with the mlp
};

struct DecoderSpec {
    std::string architecture;
    uint32_t vocab = 0, width = 0;
    float eps = 0.0f;
    NormKind norm = NormKind::Layer;
    bool norm_around_zero = false;     // norm weights are stored less one
    bool norm_scalar = false;          // norm weights are scalars
    float logit_scale = 1.0f, logit_cap = 0.0f;      // logits are scaled, then held within +-cap by a tanh (0 = not)
    bool tied_head = false;            // logits from the embedding table
    uint32_t streams = 1;              // BlockKind::Streams
    BlockKind block = BlockKind::Parallel;
    float embedding_scale = 1.0f, residual_mult = 1.0f;
    uint32_t positions = 0;        // rows of a learned position table (0 = none): the most tokens of a sequence
    std::optional<BigramSpec> bigram;
    std::vector<LayerSpec> layers;
};

inline RotationSpec read_rotation(const json::Value& v) {
    RotationSpec r;
    r.dims = v.u32("dims");
    r.base = v.num("base");
    if (const json::Value* s = v.find("scaling"); s && !s->is_null()) {
        r.scaled = true;
        r.factor = s->num("factor");
        r.original = s->num("original");
        r.fast = s->num("fast");
        r.slow = s->num("slow");
    }
    return r;
}

inline DecoderSpec read_pimosun(const json::Value& c) {
    DecoderSpec d;
    d.architecture = "Pimosun";
    d.vocab = c.u32("vocab");
    d.width = c.u32("width");
    d.eps = (float)c.at("norm").num("eps");
    if (const json::Value* e = c.find("embedding"); e && !e->is_null())
        if (const json::Value* b = e->find("bigram"); b && !b->is_null()) d.bigram = BigramSpec{b->u32("buckets"), b->u32("mul_prev"), b->u32("mul_cur")};
    const auto& layers = c.array("layers");
    for (size_t i = 0; i < layers.size(); ++i) {
        const json::Value& l = layers[i];
        const std::string where = "layer " + std::to_string(i) + ": ";
        if (l.str("type") != "latent_attention") throw json::Error(where + "unknown mixer '" + l.str("type") + "'");
        const json::Value& m = l.at("mixer");
        LayerSpec s;
        LatentAttentionSpec a;
        a.heads = m.u32("heads"); a.dim = m.u32("dim"); a.rot_dim = m.u32("rot_dim"); a.vdim = m.u32("vdim");
        a.kv_rank = m.u32("kv_rank"); a.q_rank = m.u32("q_rank");
        a.scale = (float)m.num("scale");
        a.rotation = read_rotation(m.at("rot"));
        if (const json::Value* j = m.find("kv_from"); j && !j->is_null()) a.kv_from = (int)j->as_u32("kv_from");
        if (!a.heads || !a.dim || !a.rot_dim || !a.vdim || !a.kv_rank || !a.q_rank) throw json::Error(where + "a size is zero");
        if (a.rotation.dims > a.rot_dim || a.rotation.dims % 2 != 0) throw json::Error(where + "rot.dims must be even and at most rot_dim");
        if (a.kv_from >= 0) {
            if ((size_t)a.kv_from >= i) throw json::Error(where + "kv_from must name an earlier layer");
            const LatentAttentionSpec& o = std::get<LatentAttentionSpec>(d.layers[(size_t)a.kv_from].mixer);
            if (o.kv_from >= 0 || o.kv_rank != a.kv_rank || o.rot_dim != a.rot_dim || !(o.rotation == a.rotation))
                throw json::Error(where + "kv_from must name a layer with entries of its own and the same kv_rank, rot_dim and rotation");
        }
        if (const json::Value* f = l.find("mlp"); f && !f->is_null()) {
            if (f->str("kind") != "dense") throw json::Error(where + "unknown feed-forward '" + f->str("kind") + "'");
            s.mlp = GatedMlpSpec{f->u32("ff"), Activation::GeluTanh};
            if (f->u32("ff") == 0) throw json::Error(where + "a size is zero");
        }
        s.mixer = a;
        d.layers.push_back(s);
    }
    if (d.vocab == 0 || d.width == 0 || d.layers.empty()) throw json::Error("vocab, width and layers must not be empty");
    if (d.bigram && d.bigram->buckets == 0) throw json::Error("bigram.buckets is zero");
    return d;
}

inline uint32_t optional_u32(const json::Value& v, const std::string& key, uint32_t otherwise) {
    const json::Value* f = v.find(key);
    return f && !f->is_null() ? f->as_u32(key) : otherwise;
}
inline double optional_num(const json::Value& v, const std::string& key, double otherwise) {
    const json::Value* f = v.find(key);
    return f && !f->is_null() ? v.num(key) : otherwise;
}

inline DecoderSpec read_gulidra(const json::Value& c) {
    DecoderSpec d;
    d.architecture = "Gulidra";
    d.vocab = c.u32("vocab");
    d.width = c.u32("width");
    d.eps = (float)c.at("norm").num("eps");
    d.norm = NormKind::Rms;
    d.block = BlockKind::OutputNorm;
    d.positions = c.u32("max_positions");
    d.residual_mult = (float)optional_num(c, "residual_mult", 1.0);
    if (const json::Value* e = c.find("embedding"); e && !e->is_null()) d.embedding_scale = (float)optional_num(*e, "scale", 1.0);
    const auto& layers = c.array("layers");
    for (size_t i = 0; i < layers.size(); ++i) {
        const json::Value& l = layers[i];
        const std::string where = "layer " + std::to_string(i) + ": ";
        auto check = [&](bool ok, const char* what) { if (!ok) throw json::Error(where + what); };
        const json::Value& m = l.at("mixer");
        LayerSpec s;
        if (l.str("type") == "attention") {
            DifferentialAttentionSpec a;
            a.heads = m.u32("heads"); a.kv_heads = m.u32("kv_heads"); a.dim = m.u32("dim"); a.vdim = m.u32("vdim");
            a.taps = optional_u32(m, "conv", 0);
            a.scale = (float)m.num("scale");
            a.diff = m.num("diff");
            check(a.heads && a.kv_heads && a.dim && a.vdim, "a size is zero");
            check(a.heads % a.kv_heads == 0, "heads must be a multiple of kv_heads");
            check(a.scale != 0.0f, "scale is zero");
            if (const json::Value* j = m.find("kv_from"); j && !j->is_null()) {
                const uint32_t from = j->as_u32("kv_from");
                check(from < i, "kv_from must name an earlier layer");
                const auto* o = std::get_if<DifferentialAttentionSpec>(&d.layers[from].mixer);
                check(o && o->kv_from < 0 && o->kv_heads == a.kv_heads && o->dim == a.dim && o->vdim == a.vdim,
                      "kv_from must name an attention layer with keys of its own and the same kv_heads, dim and vdim");
                a.kv_from = (int)from;
            }
            s.mixer = a;
        } else if (l.str("type") == "lightning") {
            LightningSpec a;
            a.heads = m.u32("heads"); a.dim = m.u32("dim"); a.vdim = m.u32("vdim");
            for (const json::Value& v : m.array("decay")) {
                check(v.kind == json::Value::Kind::Number && v.number > 0.0, "decay must be positive numbers");
                a.decay.push_back(v.number);
            }
            check(a.heads && a.dim && a.vdim, "a size is zero");
            check(a.decay.size() == a.heads, "decay must have one number a head");
            s.mixer = a;
        } else {
            throw json::Error(where + "unknown mixer '" + l.str("type") + "'");
        }
        if (const json::Value* f = l.find("mlp"); f && !f->is_null()) {
            if (f->str("kind") == "dense") {
                s.mlp = GatedMlpSpec{f->u32("ff"), Activation::Silu};
                check(f->u32("ff") != 0, "a size is zero");
            } else if (f->str("kind") == "moe") {
                const json::Value& r = f->at("router");
                ExpertMlpSpec e;
                e.experts = r.u32("experts"); e.identity = optional_u32(r, "identity", 0); e.top = r.u32("top");
                e.ff = f->at("expert").u32("ff");
                check(e.experts && e.top && e.ff, "a size is zero");
                check(e.top <= e.experts + e.identity, "router.top is larger than the number of experts");
                s.mlp = e;
            } else {
                throw json::Error(where + "unknown feed-forward '" + f->str("kind") + "'");
            }
        }
        d.layers.push_back(s);
    }
    if (d.vocab == 0 || d.width == 0 || d.positions == 0 || d.layers.empty()) throw json::Error("vocab, width, max_positions and layers must not be empty");
    return d;
}

inline AttentionSpec read_attention_sizes(const json::Value& m, const std::string& where) {
    AttentionSpec a;
    a.heads = m.u32("heads"); a.kv_heads = m.u32("kv_heads"); a.dim = m.u32("dim"); a.vdim = m.u32("vdim");
    a.scale = (float)m.num("scale");
    if (!a.heads || !a.kv_heads || !a.dim || !a.vdim) throw json::Error(where + "a size is zero");
    if (a.heads % a.kv_heads != 0) throw json::Error(where + "heads must be a multiple of kv_heads");
    if (a.scale == 0.0f) throw json::Error(where + "scale is zero");
    return a;
}

inline bool optional_flag(const json::Value& v, const std::string& key) {
    const json::Value* f = v.find(key);
    if (!f || f->is_null()) return false;
    if (f->kind != json::Value::Kind::Bool) throw json::Error("'" + key + "' is not true or false");
    return f->boolean;
}

inline DecoderSpec read_natatar(const json::Value& c) {
    DecoderSpec d;
    d.architecture = "Natatar";
    d.vocab = c.u32("vocab");
    d.width = c.u32("width");
    d.eps = (float)c.at("norm").num("eps");
    d.norm = NormKind::Rms;
    d.norm_around_zero = true;
    d.tied_head = true;
    d.block = BlockKind::Streams;
    d.streams = c.u32("streams");
    d.residual_mult = (float)optional_num(c, "residual_mult", 1.0);
    if (const json::Value* e = c.find("embedding"); e && !e->is_null()) d.embedding_scale = (float)optional_num(*e, "scale", 1.0);
    const auto& layers = c.array("layers");
    uint32_t shared_columns = 0;
    for (size_t i = 0; i < layers.size(); ++i) {
        const json::Value& l = layers[i];
        const std::string where = "layer " + std::to_string(i) + ": ";
        auto check = [&](bool ok, const char* what) { if (!ok) throw json::Error(where + what); };
        const json::Value& m = l.at("mixer");
        LayerSpec s;
        if (l.str("type") == "attention") {
            AttentionSpec a = read_attention_sizes(m, where);
            a.biases = a.projection_norm = true;
            a.share_values = optional_flag(m, "v_mix");
            if (a.share_values) {
                check(shared_columns == 0 || shared_columns == a.kv_heads * a.vdim, "layers that mix values must have equally many value columns");
                shared_columns = a.kv_heads * a.vdim;
            }
            s.mixer = a;
        } else if (l.str("type") == "parallel") {
            ParallelSpec p;
            const json::Value &left = m.at("left"), &right = m.at("right");
            p.left = read_attention_sizes(left, where);
            p.left.column_gate = true;
            p.left.rotation = read_rotation(left.at("rot"));
            check(p.left.rotation->dims <= p.left.dim && p.left.rotation->dims % 2 == 0, "rot.dims must be even and at most dim");
            p.right.heads = right.u32("heads"); p.right.dim = right.u32("dim"); p.right.vdim = right.u32("vdim");
            p.right.gate_cap = (float)right.num("gate_cap");
            check(p.right.heads && p.right.dim && p.right.vdim, "a size is zero");
            check(p.right.gate_cap > 0.0f, "gate_cap must be positive");
            p.left_scale = (float)optional_num(m, "left_scale", 1.0);
            p.right_scale = (float)optional_num(m, "right_scale", 1.0);
            s.mixer = p;
        } else if (l.str("type") == "channel_delta") {
            ChannelDeltaSpec a;
            a.heads = m.u32("heads"); a.kv_heads = m.u32("kv_heads"); a.dim = m.u32("dim"); a.vdim = m.u32("vdim"); a.taps = m.u32("conv");
            check(a.heads && a.kv_heads && a.dim && a.vdim && a.taps, "a size is zero");
            check(a.heads % a.kv_heads == 0, "heads must be a multiple of kv_heads");
            s.mixer = a;
        } else {
            throw json::Error(where + "unknown mixer '" + l.str("type") + "'");
        }
        if (const json::Value* f = l.find("mlp"); f && !f->is_null()) {
            if (f->str("kind") != "moe") throw json::Error(where + "unknown feed-forward '" + f->str("kind") + "'");
            const json::Value& r = f->at("router");
            ExpertMlpSpec e;
            e.correction = false;
            e.experts = r.u32("experts"); e.top = r.u32("top");
            e.ff = f->at("expert").u32("ff");
            e.scale = (float)optional_num(r, "scale", 1.0);
            if (const json::Value* g = r.find("groups"); g && !g->is_null()) { e.groups = g->u32("count"); e.keep = g->u32("keep"); }
            check(e.experts && e.top && e.ff && e.groups && e.keep, "a size is zero");
            check(e.experts % e.groups == 0, "router.experts must be a multiple of groups.count");
            check(e.keep <= e.groups, "groups.keep is larger than groups.count");
            check(e.top <= e.keep * (e.experts / e.groups), "router.top is larger than the number of experts to choose from");
            s.mlp = e;
        }
        d.layers.push_back(s);
    }
    if (d.vocab == 0 || d.width == 0 || d.streams == 0 || d.layers.empty()) throw json::Error("vocab, width, streams and layers must not be empty");
    return d;
}

// The layer whose tensors layer i uses, through any number of layers that use another's themselves.
inline int read_tensors_of(const std::vector<json::Value>& layers, size_t i, const std::string& where) {
    size_t at = i;
    for (size_t n = 0;; ++n) {
        const json::Value* j = layers[at].find("weights_of");
        if (!j || j->is_null()) return at == i ? -1 : (int)at;
        at = j->as_u32("weights_of");
        if (at >= layers.size() || n >= layers.size()) throw json::Error(where + "weights_of must lead to a layer with tensors of its own");
        for (const char* key : {"type", "mixer", "mlp"}) {
            const json::Value *a = layers[i].find(key), *b = layers[at].find(key);
            if ((a && !a->is_null()) != (b && !b->is_null()) || (a && b && *a != *b)) throw json::Error(where + "weights_of must name a layer of the same kind and sizes");
        }
    }
}

inline DecoderSpec read_fomunex(const json::Value& c) {
    DecoderSpec d;
    d.architecture = "Fomunex";
    d.vocab = c.u32("vocab");
    d.width = c.u32("width");
    d.eps = (float)c.at("norm").num("eps");
    d.norm = NormKind::Rms;
    d.norm_scalar = true;
    d.block = BlockKind::PreNorm;
    d.positions = c.u32("max_positions");
    d.logit_scale = (float)optional_num(c, "logit_scale", 1.0);
    d.logit_cap = (float)optional_num(c, "logit_softcap", 0.0);
    if (d.logit_cap < 0.0f) throw json::Error("logit_softcap must not be negative");
    const auto& layers = c.array("layers");
    for (size_t i = 0; i < layers.size(); ++i) {
        const json::Value& l = layers[i];
        const std::string where = "layer " + std::to_string(i) + ": ";
        auto check = [&](bool ok, const char* what) { if (!ok) throw json::Error(where + what); };
        const json::Value& m = l.at("mixer");
        LayerSpec s;
        s.tensors_of = read_tensors_of(layers, i, where);
        if (l.str("type") == "attention") {
            AttentionSpec a = read_attention_sizes(m, where);
            a.head_norm = a.distance_slopes = a.sink = true;
            a.cap = (float)optional_num(m, "softcap", 0.0);
            check(a.cap >= 0.0f, "softcap must not be negative");
            if (const json::Value* w = m.find("mask"); w && !w->is_null()) {
                a.window = w->u32("size");
                check(a.window > 0 && a.window <= 0x7fffffffu, "mask.size must be positive");
            }
            s.mixer = a;
        } else if (l.str("type") == "wkv") {
            const TimeMixingSpec a{m.u32("heads"), m.u32("dim")};
            check(a.heads && a.dim, "a size is zero");
            s.mixer = a;
        } else if (l.str("type") == "mamba2") {
            const StateSpaceSpec a{m.u32("heads"), m.u32("groups"), m.u32("state"), m.u32("vdim"), m.u32("conv"), m.u32("norm_groups")};
            check(a.heads && a.groups && a.state && a.vdim && a.taps && a.norm_groups, "a size is zero");
            check(a.heads % a.groups == 0, "heads must be a multiple of groups");
            check((uint64_t)a.heads * a.vdim % a.norm_groups == 0, "heads * vdim must be a multiple of norm_groups");
            s.mixer = a;
        } else {
            throw json::Error(where + "unknown mixer '" + l.str("type") + "'");
        }
        if (const json::Value* f = l.find("mlp"); f && !f->is_null()) {
            if (f->str("kind") == "dense") {
                s.mlp = PolyMlpSpec{f->u32("ff")};
                check(f->u32("ff") != 0, "a size is zero");
            } else if (f->str("kind") == "moe") {
                ExpertMlpSpec e;
                const json::Value &r = f->at("router"), &x = f->at("expert");
                e.correction = false;
                e.weight_input = true;
                e.score = RouterScore::Sigmoid;
                e.experts = r.u32("experts"); e.top = r.u32("top");
                e.ff = x.u32("ff");
                e.activation = Activation::LimitedGate;
                e.limit = (float)x.num("limit");
                e.alpha = 1.702f;
                check(e.experts && e.top && e.ff, "a size is zero");
                check(e.top <= e.experts, "router.top is larger than the number of experts");
                check(e.limit >= 0.0f, "expert.limit must not be negative");
                s.mlp = e;
            } else {
                throw json::Error(where + "unknown feed-forward '" + f->str("kind") + "'");
            }
        }
        d.layers.push_back(s);
    }
    if (d.vocab == 0 || d.width == 0 || d.positions == 0 || d.layers.empty()) throw json::Error("vocab, width, max_positions and layers must not be empty");
    return d;
}

// designs by the name config.json gives in "architecture"
inline const std::map<std::string, std::function<DecoderSpec(const json::Value&)>>& decoder_registry() {
    static const std::map<std::string, std::function<DecoderSpec(const json::Value&)>> r = {{"Pimosun", read_pimosun}, {"Gulidra", read_gulidra}, {"Natatar", read_natatar}, {"Fomunex", read_fomunex}};
    return r;
}
inline DecoderSpec read_decoder_spec(const std::string& config_text) {
    const json::Value c = json::parse(config_text.data(), config_text.size());
    const std::string& name = c.str("architecture");
    const auto it = decoder_registry().find(name);
    if (it == decoder_registry().end()) throw json::Error("unknown architecture '" + name + "'");
    return it->second(c);
}
inline std::string read_text_file(const std::string& path) {
    std::ifstream f(path, std::ios::binary);
    if (!f) throw std::runtime_error("failed to open \"" + path + "\"");
    std::ostringstream s;
    s << f.rdbuf();
    return s.str();
}

}  // namespace m40host
