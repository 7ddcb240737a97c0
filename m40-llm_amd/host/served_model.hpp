// What the scheduler, the C entry points and the command line need of a model, whatever its family.
#pragma once

#include <cstdint>

#include "scheduler.hpp"

namespace m40host {

class ServedModel {
public:
    virtual ~ServedModel() = default;
    virtual const char* family() const = 0;
    virtual uint32_t vocab() const = 0;
    virtual uint32_t max_seq_len() const = 0;       // most tokens one sequence may hold
    virtual uint32_t max_sequences() const = 0;
    virtual void set_mode(uint32_t mode) = 0;       // 0 plain launches, 1 fused, 2 fused + graph replay
    virtual void set_tie_guard(float guard) = 0;
    virtual SchedulerEngine scheduler_engine() = 0;
    virtual void decode_greedy(uint32_t seq, const uint32_t* prompt, uint32_t n_prompt, uint32_t n_gen, uint32_t start_pos,
                               uint32_t* ids_out, float* gaps_out) = 0;
    virtual void decode_batch_greedy(const uint32_t* seq_ids, const uint32_t* kv_lens, const uint32_t* first_tokens, uint32_t rows,
                                     uint32_t steps, uint32_t* ids_out, float* gaps_out) = 0;
    virtual void decode_batch_timed(const uint32_t* seq_ids, const uint32_t* kv_lens, const uint32_t* first_tokens, uint32_t rows,
                                    uint32_t warmup, uint32_t steps, uint32_t* ids_out, double* elapsed_ms) = 0;
    virtual bool last_timed_host_fallback() const = 0;
};

}  // namespace m40host
