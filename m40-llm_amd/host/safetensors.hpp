// Where a model's tensors come from: a safetensors file (8-byte little-endian header length, a JSON header of
// name -> {dtype, shape, data_offsets}, then the data), mapped and copied tensor by tensor; or random values of the shapes asked
// for (throughput runs without a checkpoint).
#pragma once

#include <cstring>
#include <map>
#include <memory>
#include <string>
#include <vector>

#include "../../include/m40llm.h"
#include "gguf.hpp"
#include "json.hpp"

namespace m40host {

class TensorSource {
public:
    virtual ~TensorSource() = default;
    // bf16 elements of `name` to device memory; throws where the tensor is missing, of another type or of another shape
    virtual void read_bf16(M40llmCudaContext* ctx, const std::string& name, const std::vector<uint64_t>& shape, void* d_dst) = 0;
    // the same to the host, widened
    virtual std::vector<float> read_f32(const std::string& name, const std::vector<uint64_t>& shape) = 0;
    // rows of a matrix whose size only the tensor itself gives
    virtual uint64_t rows_of(const std::string& name, uint64_t otherwise) = 0;
};

inline uint64_t tensor_elements(const std::vector<uint64_t>& shape) {
    uint64_t n = 1;
    for (uint64_t d : shape) n *= d;
    return n;
}

class SafetensorsFile : public TensorSource {
public:
    struct Entry {
        std::string dtype;
        std::vector<uint64_t> shape;
        uint64_t begin = 0, end = 0;      // within the data
    };
    explicit SafetensorsFile(const std::string& path) : file_(path, "safetensors file") {
        uint64_t len = 0;
        if (file_.size() < 8) throw json::Error("safetensors file too short");
        std::memcpy(&len, file_.data(), 8);
        if (len > file_.size() - 8) throw json::Error("safetensors header longer than the file");
        const json::Value head = json::parse(reinterpret_cast<const char*>(file_.data()) + 8, (size_t)len);
        data_ = 8 + len;
        const uint64_t bytes = file_.size() - data_;
        for (const auto& m : head.members) {
            if (m.first == "__metadata__") continue;
            Entry e;
            e.dtype = m.second.str("dtype");
            for (const auto& d : m.second.array("shape")) e.shape.push_back(d.as_u32("shape"));
            const auto& off = m.second.array("data_offsets");
            if (off.size() != 2 || off[0].kind != json::Value::Kind::Number || off[1].kind != json::Value::Kind::Number)
                throw json::Error("bad data_offsets of '" + m.first + "'");
            e.begin = (uint64_t)off[0].number; e.end = (uint64_t)off[1].number;
            if (e.begin > e.end || e.end > bytes) throw json::Error("tensor '" + m.first + "' lies outside the file");
            entries_[m.first] = std::move(e);
        }
    }
    const std::map<std::string, Entry>& entries() const { return entries_; }
    void read_bf16(M40llmCudaContext* ctx, const std::string& name, const std::vector<uint64_t>& shape, void* d_dst) override {
        const Entry& e = find(name, shape);
        if (m40llm_memcpy_h2d(ctx, d_dst, file_.data() + data_ + e.begin, e.end - e.begin) != 0)
            throw std::runtime_error("upload of tensor '" + name + "' failed");
    }
    std::vector<float> read_f32(const std::string& name, const std::vector<uint64_t>& shape) override {
        const Entry& e = find(name, shape);
        std::vector<float> out((e.end - e.begin) / 2);
        for (size_t i = 0; i < out.size(); ++i) {
            uint16_t b;
            std::memcpy(&b, file_.data() + data_ + e.begin + 2 * i, 2);
            const uint32_t u = (uint32_t)b << 16;
            std::memcpy(&out[i], &u, 4);
        }
        return out;
    }

    uint64_t rows_of(const std::string& name, uint64_t) override {
        const Entry& e = find(name);
        if (e.shape.empty() || e.shape[0] == 0 || e.shape[0] > 0xffffffffull) throw json::Error("tensor '" + name + "' has no rows");
        return e.shape[0];
    }

private:
    const Entry& find(const std::string& name) const {
        const auto it = entries_.find(name);
        if (it == entries_.end()) throw json::Error("no tensor named '" + name + "'");
        return it->second;
    }
    const Entry& find(const std::string& name, const std::vector<uint64_t>& shape) const {
        const Entry& e = find(name);
        if (e.dtype != "BF16") throw json::Error("tensor '" + name + "' is " + e.dtype + ", not BF16");
        if (e.shape != shape || e.end - e.begin != 2 * tensor_elements(shape)) throw json::Error("tensor '" + name + "' has another shape than config.json gives");
        return e;
    }
    gguf::MappedFile file_;
    uint64_t data_ = 0;
    std::map<std::string, Entry> entries_;
};

// Matrices uniform with the given standard deviation, vectors one.
class RandomTensors : public TensorSource {
public:
    RandomTensors(uint64_t seed, float std_dev) : seed_(seed), std_(std_dev) {}
    void read_bf16(M40llmCudaContext* ctx, const std::string& name, const std::vector<uint64_t>& shape, void* d_dst) override {
        (void)name;
        if (m40llm_ext_fill_random_bf16_async(ctx, d_dst, tensor_elements(shape), seed_ + 0x9e3779b97f4a7c15ull * ++count_, std_, M40LLM_STREAM_DECODE) != 0)
            throw std::runtime_error("random fill failed");
    }
    std::vector<float> read_f32(const std::string&, const std::vector<uint64_t>& shape) override {
        return std::vector<float>(tensor_elements(shape), 1.0f);
    }
    uint64_t rows_of(const std::string&, uint64_t otherwise) override { return otherwise; }

private:
    uint64_t seed_, count_ = 0;
    float std_;
};

}  // namespace m40host
