// Launches behind m40llm_ext_matrix_memory_async, m40llm_ext_channel_delta_async and m40llm_ext_time_mixing_async.
#pragma once

#include "memory_rules.hpp"

int m40_launch_memory_serial(hipStream_t stream, const M40MemoryArgs& a, M40MemoryRule rule, uint32_t act_dtype, uint32_t n_portions);
