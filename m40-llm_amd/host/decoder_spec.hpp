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

struct GatedMlpSpec {          // down(gelu_tanh(gate h) * (up h))
    uint32_t ff = 0;
};

struct BigramSpec {            // a second embedding looked up by (token before, token)
    uint32_t buckets = 0, mul_prev = 0, mul_cur = 0;
};

// A layer with one layer norm whose output both sublayers read: x += mixer(norm(x)) + mlp(norm(x)).
struct LayerSpec {
    LatentAttentionSpec mixer;
    std::optional<GatedMlpSpec> mlp;
};

struct DecoderSpec {
    std::string architecture;
    uint32_t vocab = 0, width = 0;
    float eps = 0.0f;
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
        LatentAttentionSpec& a = s.mixer;
        a.heads = m.u32("heads"); a.dim = m.u32("dim"); a.rot_dim = m.u32("rot_dim"); a.vdim = m.u32("vdim");
        a.kv_rank = m.u32("kv_rank"); a.q_rank = m.u32("q_rank");
        a.scale = (float)m.num("scale");
        a.rotation = read_rotation(m.at("rot"));
        if (const json::Value* j = m.find("kv_from"); j && !j->is_null()) a.kv_from = (int)j->as_u32("kv_from");
        if (!a.heads || !a.dim || !a.rot_dim || !a.vdim || !a.kv_rank || !a.q_rank) throw json::Error(where + "a size is zero");
        if (a.rotation.dims > a.rot_dim || a.rotation.dims % 2 != 0) throw json::Error(where + "rot.dims must be even and at most rot_dim");
        if (a.kv_from >= 0) {
            if ((size_t)a.kv_from >= i) throw json::Error(where + "kv_from must name an earlier layer");
            const LatentAttentionSpec& o = d.layers[(size_t)a.kv_from].mixer;
            if (o.kv_from >= 0 || o.kv_rank != a.kv_rank || o.rot_dim != a.rot_dim || !(o.rotation == a.rotation))
                throw json::Error(where + "kv_from must name a layer with entries of its own and the same kv_rank, rot_dim and rotation");
        }
        if (const json::Value* f = l.find("mlp"); f && !f->is_null()) {
            if (f->str("kind") != "dense") throw json::Error(where + "unknown feed-forward '" + f->str("kind") + "'");
            s.mlp = GatedMlpSpec{f->u32("ff")};
            if (s.mlp->ff == 0) throw json::Error(where + "a size is zero");
        }
        d.layers.push_back(s);
    }
    if (d.vocab == 0 || d.width == 0 || d.layers.empty()) throw json::Error("vocab, width and layers must not be empty");
    if (d.bigram && d.bigram->buckets == 0) throw json::Error("bigram.buckets is zero");
    return d;
}

// designs by the name config.json gives in "architecture"
inline const std::map<std::string, std::function<DecoderSpec(const json::Value&)>>& decoder_registry() {
    static const std::map<std::string, std::function<DecoderSpec(const json::Value&)>> r = {{"Pimosun", read_pimosun}};
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
