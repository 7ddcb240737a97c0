/*
 * m40llm C ABI, MI355X (gfx950) implementation.
 *
 * The drop-in boundary of the decode-step hot path: the `m40llm_*` symbols the
 * reference's Rust FFI block declares (src/cuda.rs:87-682) and its native side
 * defines (cuda/kernels.cu, C view in cuda/stub.c), with the same names, argument
 * meaning, stream behaviour and negative error codes.  Plain pointers and sizes
 * only.  Each declaration cites the reference definition it replaces.
 *
 * Conventions (all from the reference):
 *   - every function returns int (0 = ok, distinct negative code per failure
 *     site) or a handle (NULL = failure);
 *   - buffers are device pointers unless the name says host;
 *   - stream_kind: 0 = prefill stream, 1 = decode stream, anything else is an error
 *     (cuda/kernels.cu:287-292);
 *   - rope_layout: 0 = adjacent pairs (2i,2i+1), 1 = NeoX split half (i,i+hd/2);
 *   - weight_dtype: 0 = f16, 1 = f32;  exact_old_backing: 0 dense, 1 q8, 2 fp16-K/q4-V,
 *     3 (extension, M40LLM_EXT_OLD_BACKING_FP16_K_Q4G32_V) fp16-K with V 4-bit in groups of 32;
 *   - `_async` = enqueue on the decode stream and return; the GEMMs and
 *     f16_to_f32 / q80_to_f32 run on the prefill stream and block until done.
 *   - calls on one context are serialised by the caller (the reference holds a
 *     mutex around every FFI call, src/cuda.rs:1121-1137).
 *
 * Symbols of the reference that lie outside the decode hot path (staged / q8 /
 * lossy-summary attention modes, cuBLAS-only GEMM, persistent
 * decode prototype, telemetry readers) are exported and return their
 * "unavailable" code exactly as cuda/stub.c does (-1), so a binding that declares
 * all of them still links.  They are listed at the end of this header.
 *
 * Entry points that have no counterpart in the reference are prefixed
 * `m40llm_ext_` and say so.
 */
#ifndef M40LLM_H
#define M40LLM_H

#include <stddef.h>
#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

typedef struct M40llmCudaContext M40llmCudaContext;     /* src/cuda.rs:30-33   */
typedef struct M40llmKVCache M40llmKVCache;             /* src/cuda.rs:35-38   */
typedef struct M40llmCudaGraphExec M40llmCudaGraphExec; /* src/cuda.rs:40-42   */
typedef struct M40llmCudaEvent M40llmCudaEvent;         /* src/cuda.rs:43-45   */
typedef struct M40llmAttentionTelemetry M40llmAttentionTelemetry;

#define M40LLM_STREAM_PREFILL 0u
#define M40LLM_STREAM_DECODE 1u
#define M40LLM_ROPE_LAYOUT_ADJACENT 0u
#define M40LLM_ROPE_LAYOUT_NEOX 1u

/* ---- context, memory, streams (cuda/kernels.cu:276-514, 1245-1292, 7960ff) ---- */
M40llmCudaContext* m40llm_create_context(int device_id);                         /* kernels.cu:366-474 */
void m40llm_destroy_context(M40llmCudaContext* ctx);
int m40llm_current_device_props(char* name_buf, size_t buf_len, int* major, int* minor,
                                int* device_id);                                  /* kernels.cu:1245-1263 */
int m40llm_device_malloc(M40llmCudaContext* ctx, size_t bytes, void** out_ptr);   /* kernels.cu:302-310 */
int m40llm_device_free(M40llmCudaContext* ctx, void* ptr);                        /* kernels.cu:312-319 */
int m40llm_memcpy_h2d(M40llmCudaContext* ctx, void* dst_device, const void* src_host, size_t bytes);
int m40llm_memcpy_d2h(M40llmCudaContext* ctx, void* dst_host, const void* src_device, size_t bytes);
int m40llm_memcpy_d2d_async(M40llmCudaContext* ctx, void* dst_device, const void* src_device,
                            size_t bytes, uint32_t stream_kind);                  /* kernels.cu:337-355 */
int m40llm_validate_device_ptr(const void* ptr);                                  /* kernels.cu:357-364 */
int m40llm_upload_weights(M40llmCudaContext* ctx, const void* host_ptr, size_t num_bytes,
                          void** out_device_ptr);                                 /* kernels.cu:1268-1292 */
int m40llm_stream_synchronize(M40llmCudaContext* ctx, uint32_t stream_kind);      /* kernels.cu:476-484 */
int m40llm_stream_wait_for_stream(M40llmCudaContext* ctx, uint32_t waiting_stream_kind,
                                  uint32_t signal_stream_kind);                   /* kernels.cu:486-514 */

/* events and graphs (cuda/kernels.cu:516-680) */
int m40llm_cuda_event_create(M40llmCudaContext* ctx, M40llmCudaEvent** out_event);
int m40llm_cuda_event_record(M40llmCudaContext* ctx, M40llmCudaEvent* event, uint32_t stream_kind);
int m40llm_cuda_event_elapsed_sync(M40llmCudaContext* ctx, M40llmCudaEvent* start,
                                   M40llmCudaEvent* stop, float* elapsed_ms);
void m40llm_cuda_event_destroy(M40llmCudaEvent* event);
int m40llm_cuda_graph_begin_capture(M40llmCudaContext* ctx, uint32_t stream_kind);
int m40llm_cuda_graph_end_capture(M40llmCudaContext* ctx, uint32_t stream_kind,
                                  M40llmCudaGraphExec** out_graph);
int m40llm_cuda_graph_cancel_capture(M40llmCudaContext* ctx, uint32_t stream_kind);
int m40llm_cuda_graph_launch(M40llmCudaContext* ctx, M40llmCudaGraphExec* graph, uint32_t stream_kind);
int m40llm_cuda_graph_launch_timed_sync(M40llmCudaContext* ctx, M40llmCudaGraphExec* graph,
                                        uint32_t stream_kind, float* elapsed_ms);
void m40llm_cuda_graph_destroy(M40llmCudaGraphExec* graph);

/* ---- GEMV / GEMM: C[M,N] f32 row-major (cuda/kernels.cu:4981-5302) ------------- */
/* A f32 [M,K] x B f16 GGUF layout B[n*K + k]: the decode projection (kernels.cu:5158-5195) */
int m40llm_gemm_f32xf16_gguf_f32(M40llmCudaContext* ctx, const void* d_A_f32, const void* d_B_f16,
                                 void* d_C_f32, int M, int N, int K);
/* A f32 x B f16 row-major B[k*N + n] (kernels.cu:5106-5155) */
int m40llm_gemm_f32xf16_f32(M40llmCudaContext* ctx, const void* d_A_f32, const void* d_B_f16,
                            void* d_C_f32, int M, int N, int K);
/* A f16 x B f16 row-major -> f32 (kernels.cu:5267-5302) */
int m40llm_gemm_f16xf16_f32(M40llmCudaContext* ctx, const void* d_A_f16, const void* d_B_f16,
                            void* d_C_f32, int M, int N, int K);
/* A f16 x B f16 row-major -> f16, f32 accumulate (kernels.cu:5068-5103) */
int m40llm_gemm_f16_storage_f32_compute(M40llmCudaContext* ctx, const void* d_A, const void* d_B,
                                        void* d_C, int M, int N, int K);
/* GGUF f16 [N][K] -> f32 [K][N], then C[M,N] = A[M,K] x that operand (cuda/kernels.cu:5054-5066, 5197-5265; the
 * reference multiplies with cublasSgemm, here a plain f32 kernel).  Prefill stream; the non-async forms block. */
int m40llm_materialize_gguf_f16_to_f32_colmajor_nt(M40llmCudaContext* ctx, const void* d_B_f16,
                                                   void* d_B_f32_colmajor_nt, int N, int K);
int m40llm_gemm_f32xf32_f32(M40llmCudaContext* ctx, const void* d_A_f32, const void* d_B_f32_colmajor_nt,
                            void* d_C_f32, int M, int N, int K);
int m40llm_gemm_f32xf32_f32_async(M40llmCudaContext* ctx, const void* d_A_f32, const void* d_B_f32_colmajor_nt,
                                  void* d_C_f32, int M, int N, int K);
int m40llm_f16_to_f32(M40llmCudaContext* ctx, const void* d_in_f16, void* d_out_f32, size_t n);   /* :1129-1158 */
int m40llm_q80_to_f32(M40llmCudaContext* ctx, const void* d_in_q80, void* d_out_f32, size_t n);   /* :1160-1173 */

/* ---- elementwise, decode stream (cuda/kernels.cu:1036-1241, 7370-7546) ---------- */
int m40llm_rms_norm_f32(M40llmCudaContext* ctx, const void* d_in, void* d_out, uint32_t rows,
                        uint32_t dim, float eps);
int m40llm_rms_norm_f32_async(M40llmCudaContext* ctx, const void* d_in, void* d_out, uint32_t rows,
                              uint32_t dim, float eps);
int m40llm_rms_norm_f32_weighted(M40llmCudaContext* ctx, const void* d_in, const void* d_weight,
                                 void* d_out, uint32_t rows, uint32_t dim, float eps,
                                 uint32_t weight_dtype);
int m40llm_rms_norm_f32_weighted_async(M40llmCudaContext* ctx, const void* d_in, const void* d_weight,
                                       void* d_out, uint32_t rows, uint32_t dim, float eps,
                                       uint32_t weight_dtype);
int m40llm_rope_f32(M40llmCudaContext* ctx, void* d_q, void* d_k, uint32_t rows, uint32_t num_heads,
                    uint32_t head_dim, uint32_t past_len, float freq_base, float freq_scale);
int m40llm_rope_f32_async(M40llmCudaContext* ctx, void* d_q, void* d_k, uint32_t rows,
                          uint32_t num_heads, uint32_t head_dim, uint32_t past_len, float freq_base,
                          float freq_scale);
int m40llm_rope_f32_layout_async(M40llmCudaContext* ctx, void* d_q, void* d_k, uint32_t rows,
                                 uint32_t num_heads, uint32_t head_dim, uint32_t past_len,
                                 float freq_base, float freq_scale, uint32_t rope_layout);
int m40llm_rope_f32_inplace(M40llmCudaContext* ctx, void* d_x, uint32_t rows, uint32_t num_heads,
                            uint32_t head_dim, uint32_t past_len, float freq_base, float freq_scale);
int m40llm_rope_f32_inplace_async(M40llmCudaContext* ctx, void* d_x, uint32_t rows,
                                  uint32_t num_heads, uint32_t head_dim, uint32_t past_len,
                                  float freq_base, float freq_scale);
int m40llm_rope_f32_inplace_layout_async(M40llmCudaContext* ctx, void* d_x, uint32_t rows,
                                         uint32_t num_heads, uint32_t head_dim, uint32_t past_len,
                                         float freq_base, float freq_scale, uint32_t rope_layout);
int m40llm_rope_f32_inplace_position_dev_async(M40llmCudaContext* ctx, void* d_x, uint32_t rows,
                                               uint32_t num_heads, uint32_t head_dim,
                                               const uint32_t* past_len_dev, float freq_base,
                                               float freq_scale);
int m40llm_rope_f32_inplace_position_dev_layout_async(M40llmCudaContext* ctx, void* d_x, uint32_t rows,
                                                      uint32_t num_heads, uint32_t head_dim,
                                                      const uint32_t* past_len_dev, float freq_base,
                                                      float freq_scale, uint32_t rope_layout);
int m40llm_residual_add_f32(M40llmCudaContext* ctx, const void* d_a, const void* d_b, void* d_out, size_t n);
int m40llm_residual_add_f32_async(M40llmCudaContext* ctx, const void* d_a, const void* d_b, void* d_out, size_t n);
int m40llm_swiglu_f32(M40llmCudaContext* ctx, const void* d_gate, const void* d_up, void* d_out, size_t n);
int m40llm_swiglu_f32_async(M40llmCudaContext* ctx, const void* d_gate, const void* d_up, void* d_out, size_t n);

/* ---- KV cache (cuda/kernels.cu:5304-5543, 5793-6379) ---------------------------- */
M40llmKVCache* m40llm_kvcache_create(M40llmCudaContext* ctx, uint32_t max_seq_len,
                                     uint32_t max_batch_size, uint32_t num_heads, uint32_t head_dim);
/* Only exact_old_backing 0 (ring only), 2 (fp16-K/q4-V) and 3 allocate usable
 * storage here; backing 1 (q8) returns NULL.
 * Backing 3 has no counterpart in the reference: it is backing 2 with the old V rows held 4-bit in groups of 32
 * dimensions under an f16 scale and an f16 minimum (the V format the compressed-attention benchmark configuration
 * names; 80 bytes per token and head at head_dim 128 against 68).  Per group: d = f16((max - min) / 15),
 * m = f16(min), q = d > 0 ? clamp(lrintf((v - m) / d), 0, 15) : 0, value = fmaf(q, d, m).  Appends, evictions, the
 * block-select attention entry points and the debug read-backs take such a cache like a backing-2 cache;
 * m40llm_ext_kvcache_debug_read_raw(which = 2) returns head_dim / 32 words (bits of d | bits of m << 16) per token
 * and head instead of one f32 scale. */
#define M40LLM_EXT_OLD_BACKING_FP16_K_Q4G32_V 3u
M40llmKVCache* m40llm_kvcache_create_compressed(M40llmCudaContext* ctx, uint32_t max_seq_len,
                                                uint32_t max_batch_size, uint32_t num_heads,
                                                uint32_t head_dim, uint32_t recent_window,
                                                uint32_t block_size, uint32_t top_blocks,
                                                uint32_t representatives,
                                                uint32_t representative_policy,
                                                uint32_t exact_old_backing);
void m40llm_kvcache_destroy(M40llmKVCache* kv);
int m40llm_kvcache_reset(M40llmCudaContext* ctx, M40llmKVCache* kv);               /* :6308-6358 */
int m40llm_kvcache_append_token(M40llmCudaContext* ctx, M40llmKVCache* kv, uint32_t seq_id,
                                const void* k_dev_f16, const void* v_dev_f16);     /* :5793-5823 */
int m40llm_kvcache_append_token_f32(M40llmCudaContext* ctx, M40llmKVCache* kv, uint32_t seq_id,
                                    const void* k_dev_f32, const void* v_dev_f32);
int m40llm_kvcache_append_token_f32_async(M40llmCudaContext* ctx, M40llmKVCache* kv, uint32_t seq_id,
                                          const void* k_dev_f32, const void* v_dev_f32); /* :5837-5907 */
int m40llm_kvcache_append_token_f32_rope_k(M40llmCudaContext* ctx, M40llmKVCache* kv, uint32_t seq_id,
                                           const void* k_dev_f32, const void* v_dev_f32,
                                           uint32_t past_len, float freq_base, float freq_scale);
int m40llm_kvcache_append_token_f32_rope_k_async(M40llmCudaContext* ctx, M40llmKVCache* kv,
                                                 uint32_t seq_id, const void* k_dev_f32,
                                                 const void* v_dev_f32, uint32_t past_len,
                                                 float freq_base, float freq_scale);
int m40llm_kvcache_append_token_f32_rope_k_layout_async(M40llmCudaContext* ctx, M40llmKVCache* kv,
                                                        uint32_t seq_id, const void* k_dev_f32,
                                                        const void* v_dev_f32, uint32_t past_len,
                                                        float freq_base, float freq_scale,
                                                        uint32_t rope_layout);     /* :5976-6029 */
int m40llm_kvcache_append_token_f32_rope_k_at_async(M40llmCudaContext* ctx, M40llmKVCache* kv,
                                                    uint32_t seq_id, const void* k_dev_f32,
                                                    const void* v_dev_f32, uint32_t position,
                                                    uint32_t past_len, float freq_base,
                                                    float freq_scale);
/* dispatches to the compressed append/evict path when the cache is compressed (:6045-6093) */
int m40llm_kvcache_append_token_f32_rope_k_at_layout_async(M40llmCudaContext* ctx, M40llmKVCache* kv,
                                                           uint32_t seq_id, const void* k_dev_f32,
                                                           const void* v_dev_f32, uint32_t position,
                                                           uint32_t past_len, float freq_base,
                                                           float freq_scale, uint32_t rope_layout);
int m40llm_kvcache_append_token_f32_rope_k_compressed_at_async(M40llmCudaContext* ctx, M40llmKVCache* kv,
                                                               uint32_t seq_id, const void* k_dev_f32,
                                                               const void* v_dev_f32, uint32_t position,
                                                               float freq_base, float freq_scale);
int m40llm_kvcache_append_token_f32_rope_k_compressed_at_layout_async(
    M40llmCudaContext* ctx, M40llmKVCache* kv, uint32_t seq_id, const void* k_dev_f32,
    const void* v_dev_f32, uint32_t position, float freq_base, float freq_scale,
    uint32_t rope_layout);                                                         /* :6108-6250 */
int m40llm_kvcache_append_token_f32_rope_k_position_dev_async(M40llmCudaContext* ctx, M40llmKVCache* kv,
                                                              uint32_t seq_id, const void* k_dev_f32,
                                                              const void* v_dev_f32,
                                                              const uint32_t* position_dev,
                                                              float freq_base, float freq_scale);
int m40llm_kvcache_append_token_f32_rope_k_position_dev_layout_async(
    M40llmCudaContext* ctx, M40llmKVCache* kv, uint32_t seq_id, const void* k_dev_f32,
    const void* v_dev_f32, const uint32_t* position_dev, float freq_base, float freq_scale,
    uint32_t rope_layout);                                                         /* :6265-6306 */
/* one token as [kv_heads*head_dim] f16 K then V, host buffers (:6360-6379) */
int m40llm_kvcache_debug_read_token(M40llmCudaContext* ctx, M40llmKVCache* kv, uint32_t seq_id,
                                    uint32_t token, void* out_k_host, void* out_v_host);
/* telemetry twin of the block ranking: q-head 0 / kv-head 0 only (:6449-6677) */
int m40llm_kvcache_debug_select_old_blocks(M40llmCudaContext* ctx, const M40llmKVCache* kv,
                                           uint32_t seq_id, const void* q_dev_f32, uint32_t q_heads,
                                           uint32_t seq_len, uint32_t recent_window,
                                           uint32_t block_size, uint32_t top_blocks,
                                           uint32_t* out_blocks_host, float* out_scores_host,
                                           uint32_t* out_start_host, uint32_t* out_end_host,
                                           uint32_t* out_count, uint32_t max_out,
                                           uint32_t* out_total_old_blocks);

/* ---- attention, decode stream (cuda/kernels.cu:3837-4070, 4504-4577, 4694-4832) -- */
int m40llm_attention_last_token_f32(M40llmCudaContext* ctx, const M40llmKVCache* kv, uint32_t seq_id,
                                    const void* q_dev_f32, uint32_t seq_len, void* out_dev_f32);
int m40llm_attention_last_token_f32_gqa(M40llmCudaContext* ctx, const M40llmKVCache* kv,
                                        uint32_t seq_id, const void* q_dev_f32, uint32_t q_heads,
                                        uint32_t seq_len, void* out_dev_f32);
int m40llm_attention_last_token_f32_gqa_async(M40llmCudaContext* ctx, const M40llmKVCache* kv,
                                              uint32_t seq_id, const void* q_dev_f32, uint32_t q_heads,
                                              uint32_t seq_len, void* out_dev_f32);
int m40llm_attention_last_token_f32_gqa_seq_len_dev_async(M40llmCudaContext* ctx, const M40llmKVCache* kv,
                                                          uint32_t seq_id, const void* q_dev_f32,
                                                          uint32_t q_heads, const uint32_t* seq_len_dev,
                                                          void* out_dev_f32);
int m40llm_attention_last_token_f32_gqa_dense_recent_async(M40llmCudaContext* ctx, const M40llmKVCache* kv,
                                                           uint32_t seq_id, const void* q_dev_f32,
                                                           uint32_t q_heads, uint32_t seq_len,
                                                           uint32_t recent_window, void* out_dev_f32);
/* Variable-length batch: Q and Out packed [batch][q_heads][head_dim]; seq_ids / seq_lens are
 * device u32 arrays.  The reference accepts head_dim 64 and lengths <= 8192 only
 * (kernels.cu:4707, :4743); this implementation also takes head_dim 128 and any
 * length <= max_seq_len. */
int m40llm_attention_last_token_f32_gqa_batched(M40llmCudaContext* ctx, const M40llmKVCache* kv,
                                                const uint32_t* seq_ids_dev, const uint32_t* seq_lens_dev,
                                                uint32_t batch_size, const void* q_dev_f32,
                                                uint32_t q_heads, void* out_dev_f32);
int m40llm_attention_last_token_f32_gqa_batched_async(M40llmCudaContext* ctx, const M40llmKVCache* kv,
                                                      const uint32_t* seq_ids_dev,
                                                      const uint32_t* seq_lens_dev, uint32_t batch_size,
                                                      const void* q_dev_f32, uint32_t q_heads,
                                                      void* out_dev_f32);
/* block-select over a dense cache (reference: head_dim 64 only; 128 accepted here) */
int m40llm_attention_last_token_f32_gqa_block_select_exact_async(
    M40llmCudaContext* ctx, const M40llmKVCache* kv, uint32_t seq_id, const void* q_dev_f32,
    uint32_t q_heads, uint32_t seq_len, uint32_t recent_window, uint32_t block_size,
    uint32_t top_blocks, void* out_dev_f32);
/* block-select over the fp16-K / q4-V compressed cache, head_dim 64 or 128 */
int m40llm_attention_last_token_f32_gqa_block_select_exact_fp16_k_q4_v_old_direct_async(
    M40llmCudaContext* ctx, const M40llmKVCache* kv, uint32_t seq_id, const void* q_dev_f32,
    uint32_t q_heads, uint32_t seq_len, uint32_t recent_window, uint32_t block_size,
    uint32_t top_blocks, void* out_dev_f32);

/* ---- additions with no counterpart in the reference -------------------------------- */
/* q8_0 weights (34-byte blocks along K, GGUF order) -> C[M,N] f32.  The reference only
 * dequantises q8_0 elementwise (kernels.cu:856-867); this is that dequant followed by
 * the semantics of m40llm_gemm_f32xf16_gguf_f32.  Blocking, prefill stream. */
int m40llm_ext_gemm_f32xq80_gguf_f32(M40llmCudaContext* ctx, const void* d_A_f32, const void* d_B_q80,
                                     void* d_C_f32, int M, int N, int K);
/* The same product, asynchronous on the stream stream_kind names (0 prefill, 1 decode). */
int m40llm_ext_gemm_f32xq80_gguf_f32_async(M40llmCudaContext* ctx, const void* d_A_f32, const void* d_B_q80,
                                           void* d_C_f32, int M, int N, int K, uint32_t stream_kind);
/* out[M,d_model] = down(swiglu(gate(x), up(x))) with q8_0 matrices; d_scratch_f32 holds
 * 2*M*ffn floats.  Decode stream, asynchronous. */
int m40llm_ext_ffn_swiglu_q80_f32_async(M40llmCudaContext* ctx, const void* d_x_f32,
                                        const void* d_w_gate_q80, const void* d_w_up_q80,
                                        const void* d_w_down_q80, void* d_scratch_f32,
                                        void* d_out_f32, int M, int d_model, int ffn);
/* same contraction as m40llm_gemm_f32xf16_gguf_f32, enqueued on `stream_kind` without blocking */
int m40llm_ext_gemm_f32xf16_gguf_f32_async(M40llmCudaContext* ctx, const void* d_A_f32,
                                           const void* d_B_f16, void* d_C_f32, int M, int N, int K,
                                           uint32_t stream_kind);
/* One to three f16 weight matrices (GGUF order) applied to the same f32 activations A [M][K]: C_i [M][N_i] = A x B_i,
 * each exactly what m40llm_gemm_f32xf16_gguf_f32 computes.  The reference issues these as separate GEMMs
 * (qkv_project_f32xf16_gguf_f32_async and the gate/up pair, src/infer/forward.rs:2326-2338, 2471-2490); with many rows
 * they share one pass that splits A into f16 planes and one launch.  Unused matrix slots are NULL / 0.  Asynchronous on
 * `stream_kind`. */
int m40llm_ext_gemm_f32xf16_gguf_f32_multi_async(M40llmCudaContext* ctx, const void* d_A_f32, int M, int K, int n_mats,
                                                 const void* d_B0_f16, int N0, void* d_C0_f32, const void* d_B1_f16, int N1,
                                                 void* d_C1_f32, const void* d_B2_f16, int N2, void* d_C2_f32,
                                                 uint32_t stream_kind);
/* Per-q-head selection of the block-select path, computed by the same kernels that the
 * attention entry points run (the reference's debug selector covers q-head 0 only).
 * out_blocks_host: [q_heads][64] (0xffffffff beyond the count), out_counts_host: [q_heads],
 * out_scores_host (may be NULL): [q_heads][64]. Works on dense and compressed caches. */
int m40llm_ext_block_select_read_selection(M40llmCudaContext* ctx, const M40llmKVCache* kv,
                                           uint32_t seq_id, const void* q_dev_f32, uint32_t q_heads,
                                           uint32_t seq_len, uint32_t recent_window,
                                           uint32_t block_size, uint32_t top_blocks,
                                           uint32_t* out_blocks_host, uint32_t* out_counts_host,
                                           float* out_scores_host);
/* The fp16-K / q4-V block-select attention of up to 8 different sequences (slots) in one set of launches, so that
 * independent slots overlap on the device.  seq_ids_host / seq_lens_host are host arrays of n_slots entries;
 * q_dev_f32 and out_dev_f32 hold n_slots rows of q_heads * head_dim floats.  Same results and error codes as
 * n_slots calls of m40llm_attention_last_token_f32_gqa_block_select_exact_fp16_k_q4_v_old_direct_async. */
int m40llm_ext_attention_block_select_fp16_k_q4_v_multi_async(
    M40llmCudaContext* ctx, const M40llmKVCache* kv, uint32_t n_slots, const uint32_t* seq_ids_host,
    const uint32_t* seq_lens_host, const void* q_dev_f32, uint32_t q_heads, uint32_t recent_window, uint32_t block_size,
    uint32_t top_blocks, void* out_dev_f32);
/* Fill positions [0, seq_len) of one sequence from f16 K/V rows [seq_len][kv_heads][head_dim]
 * on the device, leaving the cache exactly as seq_len ordered appends of those (already
 * rotated) rows would: dense caches get the rows, compressed caches get old-K copies,
 * q4 V + scales for positions < seq_len - recent_window and ring rows for the rest. */
int m40llm_ext_kvcache_bulk_fill_f16(M40llmCudaContext* ctx, M40llmKVCache* kv, uint32_t seq_id,
                                     const void* k_dev_f16, const void* v_dev_f16, uint32_t seq_len);
/* Packed variable-length causal prefill attention, all f32 (cuda/kernels.cu:3749-3835, entry points :4834-4977;
 * declared src/cuda.rs:619-648; CPU restatement tests/attention_prefill_varlen.rs:27-76).
 * Q and Out: [total_q][q_heads][head_dim]; K and V: [total_kv][kv_heads][head_dim]; sequence b owns q_lens[b] query
 * tokens from q_offsets[b] and kv_lens[b] keys from kv_offsets[b] (token units, device arrays); query q_idx attends
 * keys 0 .. kv_len - q_len + q_idx.  Prefill stream.  The lengths are read back and validated on the host before the
 * launch in both forms, as in the reference; only the first form waits for the kernel.
 * -1 null argument, -2 batch 0, -3 head counts, -9 head_dim not 64 / 128, -7 read-back failed,
 * -8 a length is 0, q_len > kv_len or kv_len > 8192, or the key ranges of the sequences are not laid out one after the
 * other in batch order (kv_offsets[b + 1] >= kv_offsets[b] + kv_lens[b]: how packed batches are built; this
 * implementation packs K and V by sequence), -4 launch, allocation or 16-byte misaligned Q/K/V, -5 synchronise. */
int m40llm_attention_prefill_f32_gqa_varlen(M40llmCudaContext* ctx, const void* q_dev_f32, const void* k_dev_f32,
                                            const void* v_dev_f32, const uint32_t* q_offsets_dev,
                                            const uint32_t* kv_offsets_dev, const uint32_t* q_lens_dev,
                                            const uint32_t* kv_lens_dev, uint32_t batch_size, uint32_t q_heads,
                                            uint32_t kv_heads, uint32_t head_dim, void* out_dev_f32);
int m40llm_attention_prefill_f32_gqa_varlen_async(M40llmCudaContext* ctx, const void* q_dev_f32, const void* k_dev_f32,
                                                  const void* v_dev_f32, const uint32_t* q_offsets_dev,
                                                  const uint32_t* kv_offsets_dev, const uint32_t* q_lens_dev,
                                                  const uint32_t* kv_lens_dev, uint32_t batch_size, uint32_t q_heads,
                                                  uint32_t kv_heads, uint32_t head_dim, void* out_dev_f32);

/* m40llm_attention_prefill_f32_gqa_varlen_async for a caller that also holds the key offsets and the lengths on the host
 * (the same values as the device arrays, which the kernels read): validated from the host copies, so the call does not
 * read the device arrays back -- each read-back waits for everything enqueued so far, once per layer of a prefill.  No
 * counterpart in the reference (its launcher reads the lengths back).  Same codes; -1 also for a NULL host table. */
int m40llm_ext_attention_prefill_f32_gqa_varlen_host_tables_async(M40llmCudaContext* ctx, const void* q_dev_f32,
                                                                  const void* k_dev_f32, const void* v_dev_f32,
                                                                  const uint32_t* q_offsets_dev, const uint32_t* kv_offsets_dev,
                                                                  const uint32_t* q_lens_dev, const uint32_t* kv_lens_dev,
                                                                  const uint32_t* kv_offsets_host, const uint32_t* q_lens_host,
                                                                  const uint32_t* kv_lens_host, uint32_t batch_size,
                                                                  uint32_t q_heads, uint32_t kv_heads, uint32_t head_dim,
                                                                  void* out_dev_f32);

/* raw views of the compressed cache for tests: which = 0 old_k, 1 q4_v, 2 q4_scale, 3 recent_k,
 * 4 recent_v, 5 seq_map; copies `bytes` from byte offset `offset` to the host */
int m40llm_ext_kvcache_debug_read_raw(M40llmCudaContext* ctx, const M40llmKVCache* kv, uint32_t which,
                                      size_t offset, size_t bytes, void* out_host);
/* first index of the maximum of each row of logits [rows][n] -> out_idx_dev u32 [rows]; also
 * writes the top-1 minus top-2 gap to out_gap_dev (may be NULL).  Decode stream. */
int m40llm_ext_argmax_f32_async(M40llmCudaContext* ctx, const void* d_logits_f32, uint32_t rows,
                                size_t n, uint32_t* out_idx_dev, float* out_gap_dev);
/* DIAGNOSTIC, not part of the decode path.  Bandwidth yardstick (no counterpart in the reference): reads `bytes` (16-byte aligned start) of device memory
 * once, `workgroups` (<= 65536) workgroups of 256 threads each owning a contiguous range, and xors every 32-bit word
 * read into d_out_u32[0 .. 2047] (word = workgroup index modulo 2048; not cleared by the call).  One launch on the
 * decode stream; the benchmarks time it beside the kernels it bounds. */
int m40llm_ext_read_probe_async(M40llmCudaContext* ctx, const void* d_src, size_t bytes, uint32_t workgroups,
                                uint32_t* d_out_u32);
/* Prefill, steps between the Q/K/V projections and the attention for a packed batch of prompts, one launch instead
 * of three per token (src/infer/forward.rs:2349-2396: append_token_f32_rope_k_at_layout + rope_f32_inplace_layout on
 * the Q row + on the K row, per token).  Rows are packed sequence after sequence (sequence i holds q_lens_host[i]
 * rows); row j of sequence i is the token at position start_pos_host[i] + j (start_pos_host NULL = 0) of cache slot
 * seq_slots_host[i].  d_q [rows][q_heads][head_dim] and d_k [rows][kv_heads][head_dim] are rotated in place (f32);
 * the rotated K and d_v are cast to f16 into the cache, and the slot's length becomes start + len.  With the three
 * bias vectors (all or none) Q, K and V first receive their bias in place (the per-row residual adds of
 * forward.rs:149-160).  Bit-identical to the per-token calls.  Dense caches, at most 64 sequences, distinct slots.  Decode stream.
 * -1 null, -2 batch / slot / q_heads / layout, -3/-4 cache geometry, -5 past max_seq_len, -7 empty sequence,
 * -8 a slot named twice, -9 compressed cache, -6 launch. */
int m40llm_ext_prefill_rope_append_async(M40llmCudaContext* ctx, M40llmKVCache* kv, void* d_q_f32, void* d_k_f32,
                                         void* d_v_f32, uint32_t batch, const uint32_t* seq_slots_host,
                                         const uint32_t* q_lens_host, const uint32_t* start_pos_host, uint32_t q_heads,
                                         float freq_base, float freq_scale, uint32_t rope_layout, const void* d_bq_f32,
                                         const void* d_bk_f32, const void* d_bv_f32);
/* The same launch on the stream `stream_kind` names (0 prefill, 1 decode), so that a prefill can keep all of its launches on
 * one stream.  No counterpart in the reference (its per-token calls run on the decode stream). */
int m40llm_ext_prefill_rope_append_on_stream_async(M40llmCudaContext* ctx, M40llmKVCache* kv, void* d_q_f32, void* d_k_f32,
                                                   void* d_v_f32, uint32_t batch, const uint32_t* seq_slots_host,
                                                   const uint32_t* q_lens_host, const uint32_t* start_pos_host,
                                                   uint32_t q_heads, float freq_base, float freq_scale, uint32_t rope_layout,
                                                   const void* d_bq_f32, const void* d_bk_f32, const void* d_bv_f32,
                                                   uint32_t stream_kind);
/* Many-row projections of the packed prefill with the element-wise step before them and the residual add after them
 * folded in (src/infer/forward.rs:2300-2345, 2440-2530 issue these as rms_norm / swiglu, the GEMMs and residual_add, one
 * launch each).  The rows that enter the product are, by source_kind,
 *   0: d_a_f32 [M][K] as it is;
 *   1: what m40llm_rms_norm_f32_weighted writes for d_a_f32 with d_norm_weight (f16: norm_weight_dtype 0, f32: 1) and eps;
 *   2: what m40llm_swiglu_f32 writes for gate = d_a_f32 and up = d_a2_f32, both [M][K];
 * produced inside the pass that splits the rows into f16 planes, never written out as f32.  C_i [M][N_i] = rows x B_i (one
 * to three f16 GGUF matrices, as m40llm_ext_gemm_f32xf16_gguf_f32_multi_async); with one matrix and d_R0_f32 [M][N0] not NULL
 * C_0 = R_0 + product, what m40llm_residual_add_f32 gives (d_R0_f32 may be d_C0_f32).  Every result has the bits of
 * that sequence of calls (element-wise call, m40llm_ext_gemm_f32xf16_gguf_f32_multi_async over the same matrices, residual add).  Returns 0 when enqueued on `stream_kind`, 1 when the shapes are not the many-row kernel's (M <= 32, K not
 * a multiple of 32, an operand not 16-byte aligned) or its buffer cannot be provided -- nothing was enqueued and the caller
 * issues the separate calls -- and -1 / -2 / -3 for a NULL, an argument out of range, a launch failure. */
int m40llm_ext_prefill_gemm_fused_async(M40llmCudaContext* ctx, uint32_t source_kind, const void* d_a_f32, const void* d_a2_f32,
                                        const void* d_norm_weight, uint32_t norm_weight_dtype, float eps, int M, int K,
                                        int n_mats, const void* d_B0_f16, int N0, void* d_C0_f32, const void* d_R0_f32,
                                        const void* d_B1_f16, int N1, void* d_C1_f32, const void* d_B2_f16, int N2,
                                        void* d_C2_f32, uint32_t stream_kind);
/* embedding rows of `rows` (<= 65535) token ids held on the device (f16 table [vocab][d_model]) -> f32 [rows][d_model];
 * the row form of m40llm_ext_embed_token_dev_async (src/infer/forward.rs:2241-2250 loads them one blocking call per
 * token).  Decode stream. */
int m40llm_ext_embed_rows_async(M40llmCudaContext* ctx, const void* d_table_f16, const uint32_t* tokens_dev, uint32_t rows,
                                uint32_t vocab, uint32_t d_model, void* d_out_f32);
/* Weight-file ingestion: `num_bytes` of the file at `path`, from byte `file_offset`, into one new device allocation
 * (*out_device_ptr, released with m40llm_device_free).  Replaces read-the-file + m40llm_upload_weights
 * (src/infer/load.rs:27-40, kernels.cu:1264-1290): positional reads into two pinned staging buffers overlap the
 * copies to the device, and nothing the size of the file is held in host memory.  Blocks until the data is resident.
 * -1 null argument, -2 device / allocation, -3 copy, -6 the file cannot be opened or the range is not inside it. */
int m40llm_ext_upload_file_range(M40llmCudaContext* ctx, const char* path, uint64_t file_offset, uint64_t num_bytes,
                                 void** out_device_ptr);
/* Fused batch-1 decode-step entry points (decode stream, asynchronous).  They compute exactly what the
 * reference's per-op call sequence computes (src/infer/forward.rs:304-662), several steps per launch:
 *   steps 1-5: RMSNorm -> Q/K/V projections (+bias) -> RoPE(Q) -> d_q_out; RoPE(K) and V -> f16 append at the
 *              position (taken from position_dev when that is not NULL); dense caches only. */
int m40llm_ext_fused_norm_qkv_rope_append_async(
    M40llmCudaContext* ctx, M40llmKVCache* kv, uint32_t seq_id, const void* d_x_f32, const void* d_norm_w,
    uint32_t norm_weight_dtype, float eps, const void* d_wq_f16, const void* d_wk_f16, const void* d_wv_f16,
    const void* d_bq_f32, const void* d_bk_f32, const void* d_bv_f32, uint32_t d_model, uint32_t q_heads,
    uint32_t position, const uint32_t* position_dev, float freq_base, float freq_scale, uint32_t rope_layout, void* d_q_out_f32);
/*   steps 7-8 / 12-13: out = residual + W . a (residual may be NULL or alias out) */
int m40llm_ext_gemv_residual_f32xf16_async(M40llmCudaContext* ctx, const void* d_a_f32, const void* d_w_f16,
                                           const void* d_residual_f32, void* d_out_f32, int N, int K);
/*   steps 9-11: hid = silu(Wgate . xn) * (Wup . xn), xn = RMSNorm(x) * w */
int m40llm_ext_fused_norm_gate_up_swiglu_async(M40llmCudaContext* ctx, const void* d_x_f32, const void* d_norm_w,
                                               uint32_t norm_weight_dtype, float eps, const void* d_wgate_f16,
                                               const void* d_wup_f16, void* d_hid_f32, int ffn, int d_model);
/*   output norm + lm_head (src/infer/logits.rs:57-116 without the copy to the host) */
/*   With d_block_top2 (3 planes of top2_capacity 4-byte entries: largest, second largest, first index of the
 *   largest, one entry per workgroup) the kernel also leaves per-workgroup top-2 candidates for
 *   m40llm_ext_greedy_step_async; *out_n_blocks (host) receives the number of entries. */
int m40llm_ext_fused_norm_gemv_f32xf16_async(M40llmCudaContext* ctx, const void* d_x_f32, const void* d_norm_w,
                                             uint32_t norm_weight_dtype, float eps, const void* d_w_f16,
                                             void* d_out_f32, int N, int K, void* d_block_top2,
                                             uint32_t top2_capacity, uint32_t* out_n_blocks);
/* attention with the length taken from the device: seq_len = *position_dev + 1 <= max_len_hint (the launch is sized
 * for max_len_hint tokens: with a longer sequence nothing is written) */
int m40llm_ext_attention_last_token_f32_gqa_position_dev_async(M40llmCudaContext* ctx, const M40llmKVCache* kv,
                                                               uint32_t seq_id, const void* q_dev_f32,
                                                               uint32_t q_heads, const uint32_t* position_dev,
                                                               uint32_t max_len_hint, void* out_dev_f32);
/* embedding row of the token id stored at token_dev (f16 table [vocab][d_model]) -> f32 */
/* No counterpart in the reference.  m40llm_attention_last_token_f32_gqa_async for callers that cannot allocate:
 * code under HIP graph capture, tight serving loops, harnesses that forbid hipMalloc.  Same argument checks, kernels
 * and results as that entry point, but the chunk partials of rows longer than 512 tokens go into a fixed 2 MiB
 * device array that is part of the library's code object (one copy per GPU, resolved once per device when a context
 * is created), and the call allocates nothing.  Returns -9 when the partials of this (q_heads, head_dim, seq_len) do
 * not fit 2 MiB: q_heads * chunks * (head_dim + 2) * 4 bytes, chunks = ceil(seq_len / chunk) with the chunk length
 * the allocating entry point uses.  Every call on one GPU shares that array: calls on the decode stream of one context
 * are ordered and safe; a call from another context while the last user's launches are still outstanding returns -10
 * (busy) instead of racing.  Captured calls are not guarded (no event can be queried under capture): graph replays
 * that overlap on one GPU race. */
int m40llm_ext_attention_last_token_f32_gqa_static_scratch_async(M40llmCudaContext* ctx, const M40llmKVCache* kv,
                                                                 uint32_t seq_id, const void* q_dev_f32,
                                                                 uint32_t q_heads, uint32_t seq_len,
                                                                 void* out_dev_f32);
int m40llm_ext_embed_token_dev_async(M40llmCudaContext* ctx, const void* d_table_f16, const uint32_t* token_dev,
                                     uint32_t vocab, uint32_t d_model, void* d_out_f32);
/* device-side greedy step over logits[n] (scanned directly, or through the per-workgroup candidates in
 * d_block_top2): state_dev = {position, step, token, capacity, ids[capacity], gaps[capacity] (f32 bits)}; stores
 * the first index of the maximum and the top-1/top-2 gap at [step], sets token, increments step and position.
 * With d_table_f16 (f16 [n][d_model]) the embedding row of the picked token is written to d_x_out_f32. */
int m40llm_ext_greedy_step_async(M40llmCudaContext* ctx, const void* d_logits_f32, uint32_t n,
                                 const void* d_block_top2, uint32_t top2_capacity, uint32_t n_blocks,
                                 uint32_t* state_dev, const void* d_table_f16, uint32_t d_model, void* d_x_out_f32);
/* Fused row-batched decode step (1 <= rows <= 16, decode stream, asynchronous; dense caches, f16 weights, K a
 * multiple of 256).  They compute what the reference's row-batched sequence computes (src/infer/forward.rs:1729-2140),
 * several steps per call, on the MFMA skinny GEMM.  seq_lens_dev[row] is the number of tokens the row's cache holds
 * before the step (= the position of the new token); ids and lengths are read on the device only.
 *   RMSNorm -> Q/K/V projections (+bias) -> RoPE at each row's position -> q; K, V -> f16 cache rows */
int m40llm_ext_batched_norm_qkv_rope_append_async(
    M40llmCudaContext* ctx, M40llmKVCache* kv, const uint32_t* seq_ids_dev, const uint32_t* seq_lens_dev, uint32_t rows,
    const void* d_x_f32, const void* d_norm_w, uint32_t norm_weight_dtype, float eps, const void* d_wq_f16,
    const void* d_wk_f16, const void* d_wv_f16, const void* d_bq_f32, const void* d_bk_f32, const void* d_bv_f32,
    uint32_t d_model, uint32_t q_heads, float freq_base, float freq_scale, uint32_t rope_layout, void* d_q_out_f32);
/*   attention of every row over seq_lens_dev[row] + len_bias tokens (no host-side validation: rows with an id or
 *   length out of range are skipped); max_len_hint >= every row's length: the launch is sized for it, and a row
 *   that is longer is skipped like one out of range */
int m40llm_ext_attention_last_token_f32_gqa_batched_lens_dev_async(M40llmCudaContext* ctx, const M40llmKVCache* kv,
                                                                   const uint32_t* seq_ids_dev,
                                                                   const uint32_t* seq_lens_dev, uint32_t len_bias,
                                                                   uint32_t batch_size, uint32_t max_len_hint,
                                                                   const void* q_dev_f32, uint32_t q_heads,
                                                                   void* out_dev_f32);
/*   out[rows][N] = residual + a[rows][K] . W^T (residual may be NULL or alias out) */
int m40llm_ext_batched_gemm_residual_f32xf16_async(M40llmCudaContext* ctx, const void* d_a_f32, const void* d_w_f16,
                                                   const void* d_residual_f32, void* d_out_f32, uint32_t rows, int N, int K);
/*   hid[rows][ffn] = silu(gate(xn)) * up(xn), xn = RMSNorm(x) * w */
int m40llm_ext_batched_norm_gate_up_swiglu_async(M40llmCudaContext* ctx, const void* d_x_f32, const void* d_norm_w,
                                                 uint32_t norm_weight_dtype, float eps, const void* d_wgate_f16,
                                                 const void* d_wup_f16, void* d_hid_f32, uint32_t rows, int ffn, int d_model);
/*   the same, and clear_floats floats at d_clear_f32 are set to zero on the side (the result of a following
 *   ..._onto_zero call; d_clear_f32 NULL: nothing is cleared) */
int m40llm_ext_batched_norm_gate_up_swiglu_clear_async(M40llmCudaContext* ctx, const void* d_x_f32, const void* d_norm_w,
                                                       uint32_t norm_weight_dtype, float eps, const void* d_wgate_f16,
                                                       const void* d_wup_f16, void* d_hid_f32, uint32_t rows, int ffn,
                                                       int d_model, void* d_clear_f32, uint32_t clear_floats);
/*   out[rows][N] = residual + a[rows][K] . W^T for an out that HOLDS ZEROS stored by an earlier call on the decode
 *   stream (the ..._clear call above) and overlaps neither a nor residual: with rows <= 8, a long K and few columns (the
 *   down projection) one launch whose workgroups add the two halves of K into out -- two terms onto zero, the same
 *   bits in either order; any other shape falls to m40llm_ext_batched_gemm_residual_f32xf16_async, which overwrites */
int m40llm_ext_batched_gemm_residual_onto_zero_f32xf16_async(M40llmCudaContext* ctx, const void* d_a_f32, const void* d_w_f16,
                                                             const void* d_residual_f32, void* d_out_f32, uint32_t rows, int N,
                                                             int K);
/*   out[rows][N] = (RMSNorm(x) * w) . W^T  (output norm + lm_head) */
int m40llm_ext_batched_norm_gemm_f32xf16_async(M40llmCudaContext* ctx, const void* d_x_f32, const void* d_norm_w,
                                               uint32_t norm_weight_dtype, float eps, const void* d_w_f16, void* d_out_f32,
                                               uint32_t rows, int N, int K);
/*   per row: first index of the maximum of logits[row][n] and the top-1/top-2 gap -> ids_dev/gaps_dev[row][step of the
 *   row] (row stride = capacity); seq_lens_dev[row] += 1; embedding row of the pick -> d_x_out_f32[row].
 *   state_dev = {unused, capacity, step of row 0, step of row 1, ...} */
int m40llm_ext_batched_greedy_step_async(M40llmCudaContext* ctx, const void* d_logits_f32, uint32_t rows, uint32_t n,
                                         uint32_t* state_dev, uint32_t* seq_lens_dev, uint32_t* ids_dev, float* gaps_dev,
                                         const void* d_table_f16, uint32_t d_model, void* d_x_out_f32);
const char* m40llm_ext_build_info(void);

/* ---- layered decoders: bf16 weights, bf16 or f32 activations ----------------------------------------------------------------
 * Building blocks of decoders that are described layer by layer (no counterpart in the reference).  All of them are
 * asynchronous on the stream stream_kind names.  act_dtype: 0 = bf16 activations (f32 sums), 1 = f32 throughout (products
 * on the f32 matrix instruction).  Weights are bf16 in packed tiles: a [N][K] matrix is ceil(N/16) x ceil(K/32) tiles of
 * 512 elements, row tile after row tile, zero past the matrix; the element order inside a tile is the operand order of
 * the 16x16x32 matrix instruction.  "Packed" activations ([rows][ld], ld a multiple of 32) lie in the same tiles, their
 * memory a multiple of 16 rows. */
#define M40LLM_ACT_BF16 0u
#define M40LLM_ACT_F32 1u
/* Source element (nb, n, kb, k) = src[nb*sn_block + n*sn + kb*sk_block + k*sk] goes to packed row
 * n_offset + nb*n_block_pad + n and packed column k_offset + kb*k_block_pad + k of a matrix with k_tiles tiles per row
 * tile; row tile t of that counting is stored as row tile tile_first + t*tile_stride.  dst must have been cleared. */
typedef struct M40llmPackPlan {
    uint32_t n_blocks, n, n_block_pad, n_offset;
    uint32_t k_blocks, k, k_block_pad, k_offset;
    uint64_t sn_block, sn, sk_block, sk;
    uint32_t k_tiles, tile_first, tile_stride;
} M40llmPackPlan;
int m40llm_ext_pack_tiles_async(M40llmCudaContext* ctx, const void* d_src_bf16, void* d_dst, const M40llmPackPlan* plan,
                                uint32_t stream_kind);
/* n bf16 values, uniform with mean 0 and the given standard deviation, from a counter-based generator */
int m40llm_ext_fill_random_bf16_async(M40llmCudaContext* ctx, void* d_dst, uint64_t n, uint64_t seed, float std_dev,
                                      uint32_t stream_kind);
/* clears n 32-bit words with a kernel */
int m40llm_ext_clear_u32_async(M40llmCudaContext* ctx, void* d_dst, size_t n, uint32_t stream_kind);

/* what a packed product does with its sums */
#define M40LLM_PACKED_STORE 0u      /* out_f32[row][col] = v */
#define M40LLM_PACKED_ADD 1u        /* out_f32[row][col] += v */
#define M40LLM_PACKED_STORE_ACT 2u  /* out_act[row][col] = v */
#define M40LLM_PACKED_GATED 3u      /* out_act[row][batch*act_batch + col] = v * sigmoid(gate[row][batch]), packed */
#define M40LLM_PACKED_ROTATE 4u     /* heads of [plain | rotated] columns: pairs (2i, 2i+1) of the rotated part are rotated;
                                       out_act packed, rot_out (rows below split_row) plain */
#define M40LLM_PACKED_PROJECT 5u    /* the first plain_tiles tiles: as STORE; then pairs of tiles (gate, up):
                                       out_act[row][act_col + 16*pair + c] = activation(gate) * up, packed */
/* bf16, rows read from cache pages (a = the layer's cache, pages = page numbers, rows = 64 * their number):
 * KEYS: out_act = the result as a packed operand, 16-row tile after 16-row tile of n_tiles/2 k tiles;
 * VALUES: out_act = the result transposed, per page and column tile two operand tiles [16 columns][32 rows], row
 * 16t + 4g + r of 32 at place 8g + 4t + r (the order of m40llm_ext_head_attention_async) */
#define M40LLM_PACKED_KEYS 6u
#define M40LLM_PACKED_VALUES 7u
#define M40LLM_PACKED_SILU 8u       /* the first plain_tiles tiles: as STORE; then out_act[row][act_col + col] = silu(v), packed */
#define M40LLM_PACKED_SPLIT 9u      /* the same without silu */
#define M40LLM_PACKED_TANH 10u      /* the same with tanh */
#define M40LLM_PACKED_CAP 11u       /* as STORE, v = out_cap * tanh(v * out_scale / out_cap), or v * out_scale where out_cap is 0 */
#define M40LLM_GELU_TANH 0u
#define M40LLM_SILU 1u
#define M40LLM_LIMITED_GATE 2u      /* for PROJECT, with g = min(gate, act_limit), u = up held within +-act_limit: g * sigmoid(act_alpha*g) * (u + 1) */
typedef struct M40llmPackedGemm {
    uint32_t act_dtype, epilogue;
    const void* a;                /* packed [rows][lda] activations */
    uint64_t lda, a_batch;        /* columns, multiples of 32 */
    const void* w;
    uint32_t n_tiles, k_tiles;
    uint64_t w_batch;             /* elements */
    uint32_t rows, batches;
    void* out_f32;
    uint64_t ld_out, out_batch;
    void* out_act;
    uint64_t ld_act, act_batch;
    uint32_t cols, plain_tiles, act_col;
    const void* gate;
    uint64_t ld_gate;
    uint32_t head_width, rot_start, heads, split_row, rot_half;
    const void* angles;
    void* rot_out;
    uint64_t ld_rot;
    uint32_t k_parts;             /* STORE: K in that many parts, part p's sums at out_f32 + p*out_batch (0, 1 = whole) */
    const uint32_t* pages;        /* KEYS, VALUES: device */
    uint32_t page_k_tiles;        /* k tiles of a cache entry */
    uint32_t activation;          /* PROJECT: M40LLM_GELU_TANH or M40LLM_SILU */
    /* Products per expert (jobs not NULL; PROJECT without plain tiles, with `gather` up to 64 rows a job and without for 128; STORE_ACT): job j of the jobs[0] jobs behind word 4 is {expert,
     * first slot, slots}, slots at most job_rows (16, 32, 64 or 128); weights of expert e start at w + e*w_batch.  With `gather`, the
     * rows of a are plain rows gather[slot] of lda columns; without, packed rows `slot`.  Results are rows `slot`. */
    const uint32_t *jobs, *gather;
    uint32_t max_jobs, job_rows;
    const void* row_scale;        /* PROJECT: f32 [rows] (or slots), gate and up are multiplied by it before the activation; NULL = ones */
    float act_alpha, act_limit, out_scale, out_cap;
    uint32_t segment_tiles;       /* column tile t reads columns t / segment_tiles * a_batch on of a (0 = all read the same; else a multiple of 16, one batch) */
} M40llmPackedGemm;
int m40llm_ext_packed_gemm_async(M40llmCudaContext* ctx, const M40llmPackedGemm* g, uint32_t stream_kind);

/* x[row] = table[token] (+ pair_table[(prev*mul_prev + token*mul_cur) mod buckets], row `buckets` where prev is
 * 0xffffffff = the token opens its sequence; pair_table NULL = none).  bf16 tables, f32 rows. */
int m40llm_ext_embed_pairs_async(M40llmCudaContext* ctx, const void* d_table_bf16, const void* d_pair_table_bf16,
                                 const uint32_t* d_tokens, const uint32_t* d_prev, uint32_t rows, uint32_t vocab, uint32_t width,
                                 uint32_t buckets, uint32_t mul_prev, uint32_t mul_cur, void* d_x_f32, uint32_t stream_kind);
/* out[r] = layer norm of x[row_index ? row_index[r] : r] (mean taken off, eps inside the root, weight, no bias), packed;
 * out has ld_out columns, those past width zero.  n_planes > 0: x first takes the sum of as many planes of f32 rows, plane_stride
 * elements apart and laid out like x; without row_index x keeps it. */
int m40llm_ext_layer_norm_rows_async(M40llmCudaContext* ctx, void* d_x_f32, const void* d_planes_f32, uint32_t n_planes,
                                     uint64_t plane_stride, const void* d_w_f32, const uint32_t* d_row_index, uint32_t rows,
                                     uint32_t width, float eps, void* d_out, uint32_t ld_out, uint32_t act_dtype, uint32_t stream_kind);
/* angles[row][i] = (cos, sin)(position * freq[i]) * magnitude for i < pairs, (1, 0) for pairs <= i < ld_pairs; the angle is
 * formed in double precision */
int m40llm_ext_rotation_angles_async(M40llmCudaContext* ctx, const uint32_t* d_positions, uint32_t rows, const double* d_freq,
                                     uint32_t pairs, uint32_t ld_pairs, float magnitude, void* d_angles, uint32_t stream_kind);

/* The same with a scale on the token's row and a learned row per position; pair and position tables may be NULL.  h (may be NULL)
 * takes the row as a packed operand of ld_h columns, zero past width. */
typedef struct M40llmEmbedTokens {
    uint32_t act_dtype, rows, vocab, width;
    const void *table, *pair_table, *pos_table;      /* bf16 */
    const uint32_t *tokens, *prev, *positions;
    uint32_t buckets, mul_prev, mul_cur, n_positions;
    float scale;
    void* x;
    void* h;
    uint32_t ld_h;
} M40llmEmbedTokens;
int m40llm_ext_embed_tokens_async(M40llmCudaContext* ctx, const M40llmEmbedTokens* e, uint32_t stream_kind);
#define M40LLM_NORM_LAYER 0u
#define M40LLM_NORM_RMS 1u
/* m40llm_ext_layer_norm_rows_async, or with norm_kind M40LLM_NORM_RMS x / sqrt(mean(x^2) + eps) * w */
int m40llm_ext_norm_rows_async(M40llmCudaContext* ctx, uint32_t norm_kind, void* d_x_f32, const void* d_planes_f32, uint32_t n_planes,
                               uint64_t plane_stride, const void* d_w_f32, const uint32_t* d_row_index, uint32_t rows, uint32_t width,
                               float eps, void* d_out, uint32_t ld_out, uint32_t act_dtype, uint32_t stream_kind);
/* The end of a sublayer with a norm on its output: x[row] += mult * y / sqrt(mean(y^2) + eps) * w.  y is the sum of n_planes planes of f32
 * rows, plane_stride elements apart, or, where place is not NULL, sum_j weight[row*top + j] * r_j with r_j = row place[row*top + j] of
 * expert_out, or x[row] itself where place is M40LLM_PLACE_INPUT.  The new row also goes to h (packed, ld_h columns, zero past width)
 * and, where h_rows is not NULL, to plain rows of ld_h columns. */
#define M40LLM_PLACE_INPUT 0xffffffffu
typedef struct M40llmNormAdd {
    uint32_t act_dtype, rows, width;
    float eps, mult;
    void* x;
    const void* planes;
    uint32_t n_planes, top;
    uint64_t plane_stride;
    const void* expert_out;          /* act type */
    uint64_t ld_expert;
    const uint32_t* place;
    const void* weight;              /* f32 */
    const void* w;
    void *h, *h_rows;
    uint32_t ld_h;
} M40llmNormAdd;
int m40llm_ext_norm_add_rows_async(M40llmCudaContext* ctx, const M40llmNormAdd* n, uint32_t stream_kind);
/* out[row][c] = y / sqrt(mean(y^2) + eps) * w[c] * sigmoid(gate[row][c]), packed, ld_out columns, zero past cols (f32 rows y, gate) */
int m40llm_ext_norm_gate_rows_async(M40llmCudaContext* ctx, const void* d_y, uint64_t ld_y, const void* d_w, const void* d_gate,
                                    uint64_t ld_gate, uint32_t rows, uint32_t cols, float eps, void* d_out, uint32_t ld_out,
                                    uint32_t act_dtype, uint32_t stream_kind);

/* ---- routed feed-forwards ------------------------------------------------------------------------------------------------------
 * Of `experts` + `identity` experts each row takes the `top` with the largest score + correction (the lower index of equals), scores being
 * softmax(logits) or, with M40LLM_SCORE_SIGMOID, sigmoid(logits) of each; its weights are the scores times scale; slot_weight (f32 by slot, may be
 * NULL) takes them in the order of the list, for experts whose input is weighted.  groups > 1: experts form that many groups of neighbours, and only those of the `keep` groups
 * with the largest choice can be taken.  ids / weight: [rows][top].  Then rows are sorted by expert: every expert's rows, in order, take
 * slots from a multiple of 16 on; rows_of[slot] = row (slots that pad a group of 16 repeat a row), place[row*top + j] = slot, or
 * M40LLM_PLACE_INPUT for identity experts; jobs (m40llm_ext_packed_gemm_async) of at most job_rows slots; jobs[1] = slots in use.  rows_of holds
 * m40llm_ext_expert_slots, jobs 4 + 4 * m40llm_ext_expert_max_jobs words. */
#define M40LLM_SCORE_SOFTMAX 0u
#define M40LLM_SCORE_SIGMOID 1u
typedef struct M40llmRoute {
    uint32_t rows, experts, identity, top, job_rows, groups, keep, score;
    float scale;
    const void* logits;              /* f32 [rows][ld_logits] */
    uint64_t ld_logits;
    const void* correction;          /* f32 [experts + identity], NULL = none */
    uint32_t* ids;
    void* weight;                    /* f32 */
    uint32_t *rows_of, *place, *jobs;
    void* slot_weight;
} M40llmRoute;
int m40llm_ext_route_rows_async(M40llmCudaContext* ctx, const M40llmRoute* r, uint32_t stream_kind);
/* dst, packed rows of ld columns: slot s = plain row rows_of[s] of src (bf16), for the slots in use; max_slots: m40llm_ext_expert_slots */
int m40llm_ext_gather_rows_async(M40llmCudaContext* ctx, const void* d_src_bf16, uint32_t ld, const uint32_t* d_rows_of, const uint32_t* d_jobs,
                                 uint32_t max_slots, void* d_dst_bf16, uint32_t stream_kind);
uint32_t m40llm_ext_expert_slots(uint32_t rows, uint32_t experts, uint32_t top);
uint32_t m40llm_ext_expert_max_jobs(uint32_t rows, uint32_t experts, uint32_t top, uint32_t job_rows);
#define M40LLM_MAX_EXPERTS 1024u

/* ---- attention over a paged cache of keys and values, one or two maps a head -------------------------------------------------
 * One map (maps = 1): softmax attention, its result times out_scale and, where gate is not NULL, times sigmoid(gate[row][head*vdim + d]).
 * Its scores may be capped, s = cap * tanh(q.k * scale / cap) (cap 0 = not), lose slopes[head] * (distance of key and query) (f32, NULL = nothing),
 * be limited to the `window` newest tokens (0 = all), and share the denominator with a sink, exp(sink[head]) (f32, NULL = none).
 * Two maps, differential attention: softmaxes of their own queries and keys over the same values, a1 and a2; o = a1 - lambda*a2, then
 * o / sqrt(mean(o^2) + eps) * out_scale * sigmoid(gate[row][head]).  Query head h uses kv head h / (heads / kv_heads).
 * A page holds 64 tokens; per kv head first the keys, map after map (`maps` of them), as packed rows (4 x k_tiles tiles of 16 tokens x 32 dimensions),
 * then the values transposed: per 16 dimensions two tiles [16 dimensions][32 tokens], token 16t + 4g + r at place 8g + 4t + r.
 * k_tiles = dim/32, v_tiles = vdim/16, rounded up; page p starts at element p * m40llm_ext_pair_page_elements. */
uint64_t m40llm_ext_pair_page_elements(uint32_t maps, uint32_t kv_heads, uint32_t dim, uint32_t vdim);
/* From projected rows (f32: heads of [map 1 | map 2] query columns, or of one map; the same for keys, value columns): causal convolution of `taps` taps
 * on every column (0 = none), RMS norm over each map's dim of queries and keys; queries out as plain rows [heads][maps][32*k_tiles], keys and
 * values to the row's place in the cache (cache NULL = the layer reads another layer's: no key and value columns).
 * row_back[row]: rows of the same portion before it, bit 31 set where the portion is one row.  conv_state [slot][taps - 1][ld_state]
 * holds the columns of the rows before a portion, that of position p at entry p % (taps - 1) (rows before position 0 count as zero);
 * portions of one row update it, the others by m40llm_ext_conv_state_async afterwards. */
typedef struct M40llmPairSplit {
    uint32_t act_dtype, rows, maps, heads, kv_heads, dim, vdim, taps;
    float eps;
    const void* proj;
    uint64_t ld_proj;
    uint32_t k_offset, v_offset;            /* columns; queries start at 0 */
    const void *q_conv, *k_conv, *v_conv;   /* f32 [taps][columns], the newest row's last */
    const void *q_norm, *k_norm;            /* f32 [dim] */
    void* conv_state;
    uint64_t ld_state;
    void* queries;
    void* cache;
    const uint32_t *row_slot, *row_pos, *row_back, *page_table;
    uint32_t max_pages;
} M40llmPairSplit;
int m40llm_ext_pair_split_append_async(M40llmCudaContext* ctx, const M40llmPairSplit* s, uint32_t stream_kind);
/* portions[p] = {first row, rows, slot, 0}: those of two rows and more leave the last taps - 1 of their columns in conv_state */
int m40llm_ext_conv_state_async(M40llmCudaContext* ctx, const void* d_proj, uint64_t ld_proj, uint32_t cols, uint32_t taps, void* d_conv_state,
                                uint64_t ld_state, const uint32_t* d_portions, const uint32_t* d_row_pos, uint32_t n_portions,
                                uint32_t stream_kind);
/* Query i of a kv head = row * (heads / kv_heads) + head within the group.  tiles[t] = {first query, queries}, all of one slot.
 * form 0: at most 16 queries a tile, pages divided over waves and over `splits` workgroups (partial:
 * m40llm_ext_pair_attention_partial_floats; rows first_row .. first_row + n_rows are joined by a second launch); form 1: at most tile_queries
 * (64 or 128) queries a tile, operands through LDS; f32 takes rows one by one (tiles are not used).  out packed [rows][ld_out]. */
typedef struct M40llmPairAttention {
    uint32_t act_dtype, form, maps, heads, kv_heads, dim, vdim;
    float scale, lambda, out_scale, eps;
    const void* queries;
    const void* cache;
    const void* gate;                 /* f32 */
    uint64_t ld_gate;
    const uint32_t *row_slot, *row_pos, *page_table;
    uint32_t max_pages;
    const uint32_t* tiles;
    uint32_t n_tiles, tile_queries, splits, first_row, n_rows;
    void* partial;
    uint64_t partial_floats;
    void* out;
    uint32_t ld_out;
    uint32_t window;
    float cap;
    const void *slopes, *sink;
    uint32_t even;                    /* form 1: the tiles see about equally many keys (a choice of speed only) */
    float most;                       /* with a cap: |q.k| is never larger (0 = not known) */
} M40llmPairAttention;
int m40llm_ext_pair_attention_async(M40llmCudaContext* ctx, const M40llmPairAttention* a, uint32_t stream_kind);
uint64_t m40llm_ext_pair_attention_partial_floats(uint32_t maps, uint32_t rows, uint32_t heads, uint32_t vdim, uint32_t splits);
/* most queries of a tile: 128 or 64 where form 1 is served, 16 where only form 0 is, 0 = sizes that are not served */
uint32_t m40llm_ext_pair_attention_tile_queries(uint32_t act_dtype, uint32_t maps, uint32_t dim, uint32_t vdim);

/* ---- linear attention with one decay a head: lightning attention, state space layers ---------------------------------------------
 * Per head S <- decay*S + k v^T, o = S^T q, token by token; S in f32, state[slot][head][dim][32*ceil(vdim/32)], zero before position 0.
 * qkv: packed rows of the activation type, columns: heads x 32*ceil(dim/32) queries, the same of keys, heads x 32*ceil(vdim/32) values.
 * o: f32 [rows][heads*vdim].  portions[p] = {first row, rows, slot, 0}.
 * serial: token after token (any type); chunked (bf16): over the 64-row groups of the pass that a portion touches.  chunk_base[p] = chunks
 * of the portions before it; chunks[c] = {portion, first row of the group}; scratch: m40llm_ext_lightning_scratch_bytes.
 * With step_logits the decay depends on the token (Mamba-2): d = softplus(step_logits[row][head] + step_bias[head]), S <- exp(-exp(A_log[head])*d)*S +
 * d*k v^T, o = S^T q + skip[head]*v.  Head h uses query / key head h / (heads / kv_heads) (kv_heads 0 = heads): queries and keys of kv_heads heads. */
typedef struct M40llmLightning {
    uint32_t act_dtype, chunked, heads, dim, vdim;
    const void* qkv;
    uint64_t ld_qkv;
    const void* log2_decay;           /* f32 [heads] */
    const void* decay;                /* f32 [heads] */
    void* state;
    void* o;
    uint64_t ld_o;
    const uint32_t *portions, *chunk_base, *chunks, *row_pos;
    uint32_t n_portions, n_chunks;
    void* scratch;
    uint64_t scratch_bytes;
    uint32_t kv_heads;
    const void* step_logits;          /* f32 rows */
    uint64_t ld_step;
    const void *step_bias, *A_log, *skip;        /* f32 [heads] */
} M40llmLightning;
int m40llm_ext_lightning_async(M40llmCudaContext* ctx, const M40llmLightning* l, uint32_t stream_kind);
uint64_t m40llm_ext_lightning_scratch_bytes(uint32_t n_chunks, uint32_t heads, uint32_t dim, uint32_t vdim);
/* whether heads of these sizes are served */
int m40llm_ext_lightning_serves(uint32_t dim, uint32_t vdim);

/* ---- residual streams ------------------------------------------------------------------------------------------------------------------
 * x_t <- sum_s mix[s][t] x_s + mult*share[t]*y for all streams at once, then u = sum_t take[t] x_t (take NULL = ones).  x_s: f32 rows of `width`,
 * stream s at streams_x + s*stream_stride; with x0 every stream holds the row of x0 so far.  y: the sum of n_planes planes or the experts' rows,
 * as in M40llmNormAdd; neither (n_planes 0, place NULL) = the streams stay as they are.  With w, u / sqrt(mean(u^2) + eps) * w goes to h (packed,
 * ld_h columns, zero past width) and, where it is not NULL, to plain rows h_rows; without, u goes to x_out.
 * row_index (may be NULL): only these rows, `rows` of them; discard: the streams' new values are not kept. */
#define M40LLM_MOST_STREAMS 16u
/* (experts' rows without weights, weight NULL, count once each) */
typedef struct M40llmStreamUpdate {
    uint32_t act_dtype, rows, width, streams, discard;
    float eps, mult;
    const void* x0;
    void* streams_x;
    uint64_t stream_stride;
    const void *mix, *share, *take;  /* f32 [streams][streams], [streams], [streams] */
    const void* planes;
    uint32_t n_planes, top;
    uint64_t plane_stride;
    const void* expert_out;
    uint64_t ld_expert;
    const uint32_t* place;
    const void* weight;
    const void* w;
    void *h, *h_rows, *x_out;
    uint32_t ld_h;
    const uint32_t* row_index;
} M40llmStreamUpdate;
int m40llm_ext_stream_update_async(M40llmCudaContext* ctx, const M40llmStreamUpdate* u, uint32_t stream_kind);

/* ---- row-wise steps of pre-norm layers ------------------------------------------------------------------------------------------------
 * Mixes of each token's row with the one before: out column m*ld + c = h + (h' - h)*mu[m][c] for m < mixes, packed rows of mixes*ld columns.  h: plain
 * rows of the activation type, ld columns; h' is the row before of the same portion, state[slot] (f32 rows of ld) for a portion's first,
 * zero before position 0.  mu: f32 [mixes][ld].  state takes every portion's last row. */
typedef struct M40llmTokenMix {
    uint32_t act_dtype, rows, ld, mixes;
    const void* h;
    const void* mu;
    void* state;
    void* out;
    const uint32_t *portions, *row_pos, *row_back;       /* as in M40llmLightning and M40llmPairSplit */
    uint32_t n_portions;
} M40llmTokenMix;
int m40llm_ext_token_mix_async(M40llmCudaContext* ctx, const M40llmTokenMix* m, uint32_t stream_kind);
/* Normed polynomial, in place on packed rows of ld columns (zero past cols): a N(z) + b N(z^2) + c N(z^3) + e, N(y) = y / sqrt(mean(y^2) + eps) over
 * a row's cols columns; coefficients {a, b, c, e} in act (f32) */
int m40llm_ext_poly_norm_rows_async(M40llmCudaContext* ctx, void* d_z, uint32_t ld, const void* d_act, uint32_t rows, uint32_t cols, float eps, uint32_t act_dtype,
                                    uint32_t stream_kind);
/* u = y * silu(gate) (f32 rows), then each of `groups` equal parts of cols over its own sqrt(mean(u^2) + eps), times w (f32 [cols]); packed, ld_out
 * columns, zero past cols */
int m40llm_ext_gate_group_norm_rows_async(M40llmCudaContext* ctx, const void* d_y, uint64_t ld_y, const void* d_gate, uint64_t ld_gate, const void* d_w, uint32_t rows,
                                          uint32_t cols, uint32_t groups, float eps, void* d_out, uint32_t ld_out, uint32_t act_dtype, uint32_t stream_kind);
/* Causal convolution with bias and silu over projected rows (f32) whose columns are `units` blocks: heads x vdim values, then twice kv_heads x dim
 * (keys, then queries); out: the packed rows m40llm_ext_lightning_async reads (queries, keys, values, each head padded).  conv: f32 [taps][all], the newest
 * row's last; conv_state, row_back and what follows for longer portions: M40llmPairSplit. */
typedef struct M40llmSpaceSplit {
    uint32_t act_dtype, rows, heads, kv_heads, dim, vdim, taps;
    const void* proj;
    uint64_t ld_proj;
    const void *conv, *bias;
    void* conv_state;
    uint64_t ld_state;
    void* out;
    uint64_t ld_out;
    const uint32_t *row_slot, *row_pos, *row_back;
} M40llmSpaceSplit;
int m40llm_ext_space_split_async(M40llmCudaContext* ctx, const M40llmSpaceSplit* s, uint32_t stream_kind);

/* ---- attention of one map a head: from projections to queries and cache ----------------------------------------------------------
 * From projected rows (f32: query heads from column 0, key heads from k_offset, value heads from v_offset): biases (f32, may be NULL), RMS norm over
 * all query and over all key columns (q_norm [heads*dim], k_norm [kv_heads*dim], both or neither), rotation of the first 2*rot_half dimensions of
 * every query and key head in pairs (2i, 2i+1) by angles[row][rot_half] (may be NULL), queries times q_factor.  Values: keep_values takes them (f32
 * [row][ld_values]); with first_values (laid out the same) v <- (1 - lambda) v + lambda first.  Queries out as plain rows [heads][32*k_tiles], keys and
 * values to the row's place in a cache of one map. */
typedef struct M40llmQkvSplit {
    uint32_t act_dtype, rows, heads, kv_heads, dim, vdim;
    float eps, q_factor, lambda;
    const void* proj;
    uint64_t ld_proj;
    uint32_t k_offset, v_offset;
    const void *q_bias, *k_bias, *v_bias, *q_norm, *k_norm;
    const void* angles;
    uint32_t rot_half;
    const void* first_values;
    void* keep_values;
    uint64_t ld_values;
    void* queries;
    void* cache;
    const uint32_t *row_slot, *row_pos, *page_table;
    uint32_t max_pages;
} M40llmQkvSplit;
int m40llm_ext_qkv_split_append_async(M40llmCudaContext* ctx, const M40llmQkvSplit* s, uint32_t stream_kind);

/* ---- recurrent layers with a matrix state --------------------------------------------------------------------------------------------
 * All in f32, token by token, zero before position 0.  out: packed rows of the activation type, ld_out columns, head h at
 * out_col + h*vdim: o / sqrt(mean(o^2) + eps) * norm * sigmoid(gate) * out_factor.  portions[p] = {first row, rows, slot, 0}; chunk_base, chunks as in
 * M40llmLightning; chunked (bf16): a few launches over all chunks instead of token after token; scratch: m40llm_ext_memory_scratch_bytes.
 *
 * Matrix memory: log gates i = cap*tanh((zi + i_bias)/cap), f = logsigmoid(cap*tanh((zf + f_bias)/cap)); m' = max(f + m, i); S <- exp(f + m - m') S +
 * exp(i - m') k v^T, n likewise with k alone; o = S^T q / (max(|n . q|, exp(-m')) + 1e-6), q times q_factor.  proj: f32 rows with query, key, value
 * and gate columns of all heads, gate logits i and f; norm [heads*vdim]. */
typedef struct M40llmMatrixMemory {
    uint32_t act_dtype, chunked, heads, dim, vdim;
    float cap, q_factor, eps, out_factor;
    const void* proj;
    uint64_t ld_proj;
    uint32_t q_col, k_col, v_col, g_col, i_col, f_col;
    const void *i_bias, *f_bias, *norm;
    void* state;                     /* f32 [slot][heads][m40llm_ext_matrix_memory_state_floats]: S [dim][4*ceil(vdim/4)], n, m */
    void* out;
    uint32_t ld_out, out_col;
    const uint32_t *portions, *chunk_base, *chunks, *row_pos;
    uint32_t n_portions, n_chunks;
    void* scratch;
    uint64_t scratch_bytes;
} M40llmMatrixMemory;
int m40llm_ext_matrix_memory_async(M40llmCudaContext* ctx, const M40llmMatrixMemory* m, uint32_t stream_kind);
uint64_t m40llm_ext_matrix_memory_state_floats(uint32_t dim, uint32_t vdim);

/* Delta rule with one decay per head and key channel: g = exp(-exp(A_log) softplus(za + dt_bias)), b = sigmoid(zb); S <- g S (row by row);
 * u = b (v - S^T k); S <- S + k u^T; o = S^T q.  Head h uses query / key head h / (heads / kv_heads).
 * First the split: from projected rows (f32: query heads, key heads, value heads) causal convolutions (M40llmPairSplit has conv_state, row_back and
 * what follows for longer portions), silu, queries and keys x / sqrt(sum x^2 + 1e-6), queries times q_factor; out f32 rows of the same columns. */
typedef struct M40llmDeltaSplit {
    uint32_t rows, heads, kv_heads, dim, vdim, taps;
    float q_factor;
    const void* proj;
    uint64_t ld_proj;
    const void *q_conv, *k_conv, *v_conv;
    void* conv_state;
    uint64_t ld_state;
    void* out;
    uint64_t ld_out;
    const uint32_t *row_slot, *row_pos, *row_back;
} M40llmDeltaSplit;
int m40llm_ext_delta_split_async(M40llmCudaContext* ctx, const M40llmDeltaSplit* s, uint32_t stream_kind);
typedef struct M40llmChannelDelta {
    uint32_t act_dtype, chunked, heads, kv_heads, dim, vdim;
    float q_factor, eps, out_factor;
    const void* qkv;                 /* f32 rows of the split */
    uint64_t ld_qkv;
    const void* low;                 /* f32 rows: decay logits [heads*dim] from a_col on, gate logits [heads*vdim] from g_col on */
    uint64_t ld_low;
    uint32_t a_col, g_col;
    const void* beta;                /* f32 rows of write strength logits [heads] */
    uint64_t ld_beta;
    const void *A_log, *dt_bias, *norm;      /* f32 [heads], [heads*dim], [vdim] */
    void* state;                     /* f32 [slot][heads][m40llm_ext_channel_delta_state_floats]: S [dim][4*ceil(vdim/4)] */
    void* out;
    uint32_t ld_out, out_col;
    const uint32_t *portions, *chunk_base, *chunks, *row_pos;
    uint32_t n_portions, n_chunks;
    void* scratch;
    uint64_t scratch_bytes;
} M40llmChannelDelta;
int m40llm_ext_channel_delta_async(M40llmCudaContext* ctx, const M40llmChannelDelta* m, uint32_t stream_kind);
uint64_t m40llm_ext_channel_delta_state_floats(uint32_t dim, uint32_t vdim);
/* Time mixing with a bonus (RWKV): w = exp(-exp(zw + w0)) per head and key channel; o = (S + diag(u) k v^T)^T r; then S <- diag(w) S + k v^T.
 * rkv: f32 rows, receptance, key, value and gate columns of all heads; out: o / sqrt(mean(o^2) + eps) * norm * silu(gate) * out_factor (norm [heads*dim]). */
typedef struct M40llmTimeMixing {
    uint32_t act_dtype, chunked, heads, dim;
    float eps, out_factor;
    const void* rkv;
    uint64_t ld_rkv;
    uint32_t r_col, k_col, v_col, g_col;
    const void* decay;               /* f32 rows of zw, heads*dim columns */
    uint64_t ld_decay;
    const void *w0, *u, *norm;       /* f32 [heads*dim] */
    void* state;                     /* f32 [slot][heads][m40llm_ext_channel_delta_state_floats(dim, dim)] */
    void* out;
    uint32_t ld_out, out_col;
    const uint32_t *portions, *chunk_base, *chunks, *row_pos;
    uint32_t n_portions, n_chunks;
    void* scratch;
    uint64_t scratch_bytes;
} M40llmTimeMixing;
int m40llm_ext_time_mixing_async(M40llmCudaContext* ctx, const M40llmTimeMixing* m, uint32_t stream_kind);
#define M40LLM_RULE_MEMORY 0u
#define M40LLM_RULE_DELTA 1u
#define M40LLM_RULE_MIXING 2u
uint64_t m40llm_ext_memory_scratch_bytes(uint32_t rule, uint32_t n_chunks, uint32_t heads, uint32_t dim, uint32_t vdim);
/* whether heads of these sizes are served */
int m40llm_ext_memory_serves(uint32_t dim, uint32_t vdim);

/* ---- latent attention over a paged cache ------------------------------------------------------------------------------------
 * A page holds 64 tokens; a token's entry is its normed latent (kv_rank, padded to a multiple of 32) followed by the rotated
 * key part all heads share (rot_dim, padded to a multiple of 32): entry_width elements of the activation type, in packed
 * tile order (4 x entry_width/32 tiles a page).  Page p of a layer starts at base + p*64*entry_width.  Sequence slot s
 * finds its pages in page_table[s*max_pages + position/64]. */
#define M40LLM_PAGE_TOKENS 64u
/* From the projected row [q latent | kv latent | rotated key part | ...] (f32, parts padded to multiples of 16 / 32):
 * cq[row] = RMSNorm(q latent) (packed, ld_cq columns, zero past q_rank), and where cache is not NULL RMSNorm(kv latent) and the
 * rotated key part go to the row's place in the cache. */
typedef struct M40llmLatentSplit {
    uint32_t act_dtype, rows;
    const void* proj;                 /* f32 [rows][ld_proj] */
    uint64_t ld_proj;
    uint32_t q_rank, kv_offset, kv_rank, rot_offset, rot_dim;
    const void *q_norm, *kv_norm;     /* f32 weights */
    float eps;
    void* cq;
    uint32_t ld_cq;
    void* cache;                      /* NULL = the layer reads another layer's entries */
    uint32_t latent_pad, entry_width, rot_half;
    const void* angles;
    const uint32_t *row_slot, *row_pos, *page_table;
    uint32_t max_pages;
} M40llmLatentSplit;
int m40llm_ext_latent_split_append_async(M40llmCudaContext* ctx, const M40llmLatentSplit* s, uint32_t stream_kind);
/* Attention of query rows i = row*heads + head given in latent space (queries [rows*heads][entry_width]: W_uk^T q, then the
 * rotated part): score = q . entry * scale over the positions <= row_pos[row] of the row's slot, softmax whose denominator
 * also holds exp(sink[head]), result = weighted sum of the latents, out packed [rows][heads*latent_pad].
 * tiles[t] = {first query row, query rows}: all of one slot, at most 16*m_tiles.  splits > 1 divides the pages of a tile over
 * that many workgroups; partial sums go to `partial` (m40llm_ext_latent_attention_partial_floats) and are joined by a
 * second launch. */
typedef struct M40llmLatentAttention {
    uint32_t act_dtype, heads, kv_rank, latent_pad, entry_width;
    float scale;
    const void* queries;
    const void* cache;
    const void* sink;                 /* f32 [heads] */
    const uint32_t *row_slot, *row_pos, *page_table;
    uint32_t max_pages;
    const uint32_t* tiles;            /* device, 2 words a tile */
    uint32_t n_tiles, m_tiles, splits;
    uint32_t first_query, n_queries;  /* the range the tiles cover (partials and the joining launch) */
    void* partial;
    uint64_t partial_floats;
    void* out;
} M40llmLatentAttention;
int m40llm_ext_latent_attention_async(M40llmCudaContext* ctx, const M40llmLatentAttention* a, uint32_t stream_kind);
uint64_t m40llm_ext_latent_attention_partial_floats(uint32_t n_queries, uint32_t latent_pad, uint32_t splits);
/* the largest m_tiles the kernels serve for an entry width (0 = the width is not served) */
uint32_t m40llm_ext_latent_attention_max_m_tiles(uint32_t act_dtype, uint32_t kv_rank, uint32_t entry_width);
/* The same attention for long portions, over keys and values brought out of the latents head by head.  pages: the page lists of the
 * portions one behind the other; keys / values: what M40LLM_PACKED_KEYS / _VALUES write for that list (heads of 32*plain_tiles key
 * columns, heads of 16*v_tiles value columns); the rotated key part (the last rot_tiles of a cache entry's entry_tiles) is
 * read from the cache.  queries: packed [rows][ld_queries], per head [plain | rotated].  jobs[t] = {first row, rows (at most job_rows),
 * first page of the portion's sequence in `pages`, 0}.  out[row][head*vdim + d], packed = result * sigmoid(gate[row][head]). */
typedef struct M40llmHeadAttention {
    uint32_t heads, plain_tiles, rot_tiles, entry_tiles, vdim, v_tiles;
    float scale;
    const void* queries;
    uint32_t ld_queries;
    const void *keys, *values, *cache, *sink;
    const void* gate;
    uint64_t ld_gate;
    const uint32_t *row_pos, *pages, *jobs;
    uint32_t n_jobs, job_rows;        /* job_rows: 64 or 128 */
    void* out;
    uint32_t ld_out;
} M40llmHeadAttention;
int m40llm_ext_head_attention_async(M40llmCudaContext* ctx, const M40llmHeadAttention* a, uint32_t stream_kind);
/* whether a head of as many 32-wide key tiles (plain and rotated) and 16-wide value tiles is served */
int m40llm_ext_head_attention_serves(uint32_t k_tiles, uint32_t v_tiles);
/* Largest and second largest logit of every row, in M40LLM_TOP2_PARTS parts a row: parts[row][part] = {largest, second largest,
 * first index of the largest, 0} (f32, f32, u32, u32) */
#define M40LLM_TOP2_PARTS 32u
int m40llm_ext_top2_parts_async(M40llmCudaContext* ctx, const void* d_logits_f32, uint32_t rows, uint32_t vocab, void* d_parts,
                                uint32_t stream_kind);
/* Greedy step of a device-driven decode loop: row r's token is the first index of its largest logit (from parts); it and the gap to
 * the second largest are recorded at ids[r*capacity + step] / gaps[...], it becomes the input token (prev = the token before), the
 * position advances by one.  state[0] = step counter. */
int m40llm_ext_advance_rows_async(M40llmCudaContext* ctx, const void* d_parts, uint32_t rows, uint32_t* d_tokens, uint32_t* d_prev,
                                  uint32_t* d_positions, uint32_t* d_state, uint32_t* d_ids, float* d_gaps, uint32_t capacity,
                                  uint32_t stream_kind);

/* ---- present but unavailable (return -1, as cuda/stub.c does) ---------------------- */
int m40llm_kvcache_build_q8_old_from_dense(M40llmCudaContext*, M40llmKVCache*, uint32_t, uint32_t, uint32_t);
int m40llm_kvcache_build_compressed_from_dense(M40llmCudaContext*, M40llmKVCache*, const M40llmKVCache*, uint32_t);
int m40llm_kvcache_debug_read_compressed_state(M40llmCudaContext*, M40llmKVCache*, uint32_t, uint32_t*,
                                               uint32_t*, void*, void*, float*, float*, void*, void*,
                                               void*, void*, uint32_t*);
int m40llm_kvcache_debug_attention_telemetry(M40llmCudaContext*, const M40llmKVCache*, uint32_t, uint32_t,
                                             const void*, uint32_t, uint32_t, uint32_t, uint32_t, uint32_t,
                                             uint32_t, M40llmAttentionTelemetry*);
int m40llm_attention_last_token_f32_gqa_block_select_exact_staged_async(
    M40llmCudaContext*, const M40llmKVCache*, uint32_t, const void*, uint32_t, uint32_t, uint32_t,
    uint32_t, uint32_t, void*);
int m40llm_attention_last_token_f32_gqa_block_select_exact_staged_with_buffers_async(
    M40llmCudaContext*, const M40llmKVCache*, uint32_t, const void*, uint32_t, uint32_t, uint32_t,
    uint32_t, uint32_t, void*, void*, void*, void*, uint32_t, void*);
int m40llm_attention_last_token_f32_gqa_block_select_exact_staged_q8_old_with_buffers_async(
    M40llmCudaContext*, const M40llmKVCache*, uint32_t, const void*, uint32_t, uint32_t, uint32_t,
    uint32_t, uint32_t, void*, void*, void*, void*, uint32_t, void*);
int m40llm_attention_last_token_f32_gqa_block_select_exact_staged_fp16_k_q4_v_old_with_buffers_async(
    M40llmCudaContext*, const M40llmKVCache*, uint32_t, const void*, uint32_t, uint32_t, uint32_t,
    uint32_t, uint32_t, void*, void*, void*, void*, uint32_t, void*);
int m40llm_attention_last_token_f32_gqa_block_select_exact_q8_old_direct_async(
    M40llmCudaContext*, const M40llmKVCache*, uint32_t, const void*, uint32_t, uint32_t, uint32_t,
    uint32_t, uint32_t, void*);
int m40llm_attention_last_token_f32_gqa_block_summary_lossy_async(
    M40llmCudaContext*, const M40llmKVCache*, uint32_t, const void*, uint32_t, uint32_t, uint32_t,
    uint32_t, uint32_t, void*);
int m40llm_attention_last_token_f32_gqa_compressed_recent_only_async(
    M40llmCudaContext*, const M40llmKVCache*, uint32_t, const void*, uint32_t, uint32_t, void*);
int m40llm_start_persistent_decode(M40llmCudaContext*);
int m40llm_stop_persistent_decode(M40llmCudaContext*);
int m40llm_persistent_decode_submit_vec(M40llmCudaContext*, const void*, void*, uint32_t, float, float,
                                        uint32_t, uint32_t*);
int m40llm_persistent_decode_poll(M40llmCudaContext*, uint32_t*, uint32_t*);

#ifdef __cplusplus
}
#endif
#endif /* M40LLM_H */
