/*
 * lightseq_lm.h -- C ABI of the floating-point decoder kernels (no counterpart in the reference): one
 * entry point per mechanism, each for bfloat16 (_bf16) and float32 (_f32) activations.  Pointers are
 * device pointers unless they are described as descriptors; matrices are row-major, linear weights
 * [out, in]; the residual stream, router logits, recurrent states and norm weights are float32.
 *
 * Rows of a batch are packed: sequence i of a step owns rows [row0, row0 + n), which are its
 * positions [pos0, pos0 + n), and the cache place `slot`.
 *
 * What each function computes stands with its launcher in lightseq_amd/csrc/lm_launch.h.
 */
#ifndef LIGHTSEQ_LM_H_
#define LIGHTSEQ_LM_H_

#include "lightseq_hip.h"

#ifdef __cplusplus
extern "C" {
#endif

typedef struct lsh_seq_span_t {
  int row0, n, pos0, slot;
} lsh_seq_span_t; /* arrays of it are device memory */

/* descriptors (host memory) */
typedef struct lsh_attn_shape_t {
  int heads, kv_heads, dim, vdim, max_step;
} lsh_attn_shape_t;
typedef struct lsh_attn_mask_t {
  int window, keep_first; /* position i sees j <= i with i - j < window (<= 0: any) or j < keep_first */
  float scale;
  int sink;               /* exp(sinks[head]) is added to the soft-max denominator, 1 without sinks */
  int chunk;              /* > 0: only keys of the query's own chunk of so many positions (or kept ones) */
  const float* sinks;     /* device, [heads], or null */
} lsh_attn_mask_t;
typedef struct lsh_delta_shape_t {
  int heads, kv_heads, dim, vdim, taps;
} lsh_delta_shape_t;

/* a summand of the residual row; post_w null: no norm of its own */
typedef struct lsh_residual_part_t {
  const void* y; /* null: none */
  int parts;
  int64_t part_stride, row_stride;
  const float *weight, *post_w, *post_b;
} lsh_residual_part_t;
/* x <- x + scale * (part 0 + part 1) + embed[inject_ids] + inject_vec;  h = norm(x) */
typedef struct lsh_residual_t {
  lsh_residual_part_t part[2];
  int y_is_float;          /* else the parts have the activations' type */
  int post_rms, norm_rms;  /* root-mean-square norms (no mean, no bias) instead of layer norms */
  float scale;
  const float *norm_w, *norm_b; /* norm_w null: no output */
  const int* inject_ids;        /* null: none */
  const float* inject_vec;      /* null: none */
} lsh_residual_t;
typedef struct lsh_gla_shape_t {
  int heads, dim, vdim, rank;      /* rank: a multiple of 16 */
  int q_col, k_col, v_col, g_col;  /* columns of the projection */
  float tau, eps;
} lsh_gla_shape_t;

/* row length of the key and value caches [slot][kv_head][max_step][pad]; 0: not supported */
int lsh_lm_attn_pad(int dim);
int64_t lsh_lm_attn_decode_workspace(int rows, const lsh_attn_shape_t* shape);           /* floats */
int64_t lsh_lm_delta_chunked_workspace(int rows, int n_seqs, const lsh_delta_shape_t* shape);
int lsh_lm_delta_chunked_supported(const lsh_delta_shape_t* shape);
int64_t lsh_lm_gla_chunked_workspace(int rows, int n_seqs, const lsh_gla_shape_t* shape); /* floats */
int lsh_lm_gla_chunked_supported(const lsh_gla_shape_t* shape, int64_t ld);

int lsh_lm_moe_route(const float* logits, const float* bias, float* weight, int* count, int* list,
                     int tokens, int experts, int top, lsh_stream_t stream);
int lsh_lm_sample(const float* logits, int rows, int vocab, int topk, float topp, int eos_id,
                  void* rng_state, int* ids, int max_step, int* last_ids, int* row_len, int* row_pos,
                  int* unfinished, lsh_stream_t stream);

int lsh_lm_gemm_f32(const void* A, int64_t lda, const void* W, void* C, int64_t ldc, float*
    C2, int64_t ld2, int n_split, int M, int N, int K, lsh_stream_t stream);
int lsh_lm_gemm_bf16(const void* A, int64_t lda, const void* W, void* C, int64_t ldc, float*
    C2, int64_t ld2, int n_split, int M, int N, int K, lsh_stream_t stream);
int lsh_lm_gemm_f32_out_f32(const void* A, int64_t lda, const void* W, float* C, int M, int N,
    int K, lsh_stream_t stream);
int lsh_lm_gemm_f32_out_bf16(const void* A, int64_t lda, const void* W, float* C, int M, int N,
    int K, lsh_stream_t stream);
int lsh_lm_gemm_planes_f32(const void* A, int64_t lda, const void* W, float* C, int M, int N,
    int K, int max_planes, int* planes_used, lsh_stream_t stream);
int lsh_lm_gemm_planes_bf16(const void* A, int64_t lda, const void* W, float* C, int M, int N,
    int K, int max_planes, int* planes_used, lsh_stream_t stream);
int lsh_lm_moe_router_f32(const void* h, const void* w, const float* bias, float* weight, int* count,
    int* list, int tokens, int width, int experts, int top, lsh_stream_t stream);
int lsh_lm_moe_router_bf16(const void* h, const void* w, const float* bias, float* weight, int* count,
    int* list, int tokens, int width, int experts, int top, lsh_stream_t stream);
int lsh_lm_moe_up_f32(const void* h, const void* w, void* act, const int* count, const int* list,
    int tokens, int top, int experts, int width, int ff, lsh_stream_t stream);
int lsh_lm_moe_up_bf16(const void* h, const void* w, void* act, const int* count, const int* list,
    int tokens, int top, int experts, int width, int ff, lsh_stream_t stream);
int lsh_lm_moe_down_f32(const void* act, const void* w, void* out, const int* count, const int*
    list, int tokens, int top, int experts, int width, int ff, lsh_stream_t stream);
int lsh_lm_moe_down_bf16(const void* act, const void* w, void* out, const int* count, const int*
    list, int tokens, int top, int experts, int width, int ff, lsh_stream_t stream);
int lsh_lm_norm_f32(float* x, const void* y, int y_is_float, int parts, int64_t part_stride,
    int64_t row_stride, const float* weight, const float* post_w, const float* post_b, const
    float* norm_w, const float* norm_b, void* h, int rows, int width, float eps, const int* ids,
    const void* embed, int vocab, const int* from_rows, int* zero_count, int n_zero, lsh_stream_t
    stream);
int lsh_lm_norm_bf16(float* x, const void* y, int y_is_float, int parts, int64_t part_stride,
    int64_t row_stride, const float* weight, const float* post_w, const float* post_b, const
    float* norm_w, const float* norm_b, void* h, int rows, int width, float eps, const int* ids,
    const void* embed, int vocab, const int* from_rows, int* zero_count, int n_zero, lsh_stream_t
    stream);
int lsh_lm_attn_prepare_f32(const void* proj, int64_t ld, int q_col, int k_col, int v_col, const
    float* q_norm, const float* k_norm, float eps, const float* cos_sin, int rot_pairs, void*
    q_out, void* k_cache, void* v_cache, const int* row_slot, const int* row_pos, int rows, const
    lsh_attn_shape_t* sh, lsh_stream_t stream);
int lsh_lm_attn_prepare_bf16(const void* proj, int64_t ld, int q_col, int k_col, int v_col,
    const float* q_norm, const float* k_norm, float eps, const float* cos_sin, int rot_pairs,
    void* q_out, void* k_cache, void* v_cache, const int* row_slot, const int* row_pos, int rows,
    const lsh_attn_shape_t* sh, lsh_stream_t stream);
int lsh_lm_attn_prefill_f32(const void* q, const void* k_cache, const void* v_cache, const void*
    proj, int64_t ld, int g_col, void* out, const lsh_seq_span_t* seqs, int n_seqs, int max_n,
    const lsh_attn_shape_t* sh, const lsh_attn_mask_t* mask, lsh_stream_t stream);
int lsh_lm_attn_prefill_bf16(const void* q, const void* k_cache, const void* v_cache, const void*
    proj, int64_t ld, int g_col, void* out, const lsh_seq_span_t* seqs, int n_seqs, int max_n,
    const lsh_attn_shape_t* sh, const lsh_attn_mask_t* mask, lsh_stream_t stream);
int lsh_lm_attn_decode_f32(const void* q, const void* k_cache, const void* v_cache, const void*
    proj, int64_t ld, int g_col, void* out, const int* row_slot, const int* row_pos, int rows,
    int max_len, float* workspace, const lsh_attn_shape_t* sh, const lsh_attn_mask_t* mask,
    lsh_stream_t stream);
int lsh_lm_attn_decode_bf16(const void* q, const void* k_cache, const void* v_cache, const void*
    proj, int64_t ld, int g_col, void* out, const int* row_slot, const int* row_pos, int rows,
    int max_len, float* workspace, const lsh_attn_shape_t* sh, const lsh_attn_mask_t* mask,
    lsh_stream_t stream);
int lsh_lm_delta_prepare_f32(const void* proj, int64_t ld, const float* ba, const float* conv_w,
    const float* a_log, const float* dt_bias, void* conv_ring, float* q, float* k, void* v, float*
    log_g, float* beta, const lsh_seq_span_t* seqs, int n_seqs, int max_n, const
    lsh_delta_shape_t* sh, lsh_stream_t stream);
int lsh_lm_delta_prepare_bf16(const void* proj, int64_t ld, const float* ba, const float*
    conv_w, const float* a_log, const float* dt_bias, void* conv_ring, float* q, float* k, void*
    v, float* log_g, float* beta, const lsh_seq_span_t* seqs, int n_seqs, int max_n, const
    lsh_delta_shape_t* sh, lsh_stream_t stream);
int lsh_lm_delta_scan_f32(const float* q, const float* k, const void* v, const float* log_g, const
    float* beta, float* state, float* o, const lsh_seq_span_t* seqs, int n_seqs, const
    lsh_delta_shape_t* sh, lsh_stream_t stream);
int lsh_lm_delta_scan_bf16(const float* q, const float* k, const void* v, const float* log_g,
    const float* beta, float* state, float* o, const lsh_seq_span_t* seqs, int n_seqs, const
    lsh_delta_shape_t* sh, lsh_stream_t stream);
int lsh_lm_delta_chunked_f32(const float* q, const float* k, const void* v, const float* log_g,
    const float* beta, float* state, float* o, float* workspace, const lsh_seq_span_t* seqs, int
    n_seqs, int max_n, int rows, const lsh_delta_shape_t* sh, lsh_stream_t stream);
int lsh_lm_delta_chunked_bf16(const float* q, const float* k, const void* v, const float* log_g,
    const float* beta, float* state, float* o, float* workspace, const lsh_seq_span_t* seqs, int
    n_seqs, int max_n, int rows, const lsh_delta_shape_t* sh, lsh_stream_t stream);
int lsh_lm_delta_gated_norm_f32(const float* o, const void* proj, int64_t ld, int g_col, const
    float* norm_w, float eps, void* out, int rows, const lsh_delta_shape_t* sh, lsh_stream_t
    stream);
int lsh_lm_delta_gated_norm_bf16(const float* o, const void* proj, int64_t ld, int g_col, const
    float* norm_w, float eps, void* out, int rows, const lsh_delta_shape_t* sh, lsh_stream_t
    stream);
int lsh_lm_delta_step_f32(const void* proj, int64_t ld, int g_col, const float* ba, const float*
    conv_w, const float* a_log, const float* dt_bias, const float* norm_w, float eps, void*
    conv_ring, float* state, void* out, const int* row_slot, const int* row_pos, int rows, const
    lsh_delta_shape_t* sh, lsh_stream_t stream);
int lsh_lm_delta_step_bf16(const void* proj, int64_t ld, int g_col, const float* ba, const
    float* conv_w, const float* a_log, const float* dt_bias, const float* norm_w, float eps, void*
    conv_ring, float* state, void* out, const int* row_slot, const int* row_pos, int rows, const
    lsh_delta_shape_t* sh, lsh_stream_t stream);

int lsh_lm_gemm_epilogue_f32(const void* A, int64_t lda, const void* W, void* C, int64_t ldc,
    float* C2, int64_t ld2, int n_split, int M, int N, int K, float scale, const float* bias,
    lsh_stream_t stream);
int lsh_lm_gemm_gated_f32(const void* A, int64_t lda, const void* W, void* C, int64_t ldc, int M,
    int N, int K, int act, lsh_stream_t stream); /* act 0: silu, 1: relu */
int lsh_lm_residual_f32(float* x, const lsh_residual_t* what, void* h, int rows, int width, float eps,
    const int* ids, const void* embed, int vocab, lsh_stream_t stream);
int lsh_lm_attn_decode_append_f32(const void* proj, int64_t ld, int q_col, int k_col, void* k_cache,
    void* out, const int* row_slot, const int* row_pos, int rows, int max_len, float* workspace, const
    lsh_attn_shape_t* sh, const lsh_attn_mask_t* mask, lsh_stream_t stream);
int lsh_lm_gemm_planes2_f32(const void* A0, int64_t lda0, const void* W0, float* C0, int K0, const
    void* A1, int64_t lda1, const void* W1, float* C1, int K1, int M, int N, int max_planes, int*
    planes0, int* planes1, lsh_stream_t stream);
int lsh_lm_gla_step_f32(const void* proj, int64_t ld, const float* low, const float* a2, const float*
    bias, const float* norm, float* state, void* out, const int* row_slot, const int* row_pos, int
    rows, const lsh_gla_shape_t* sh, lsh_stream_t stream);
int lsh_lm_gla_scan_f32(const void* proj, int64_t ld, const float* low, const float* a2, const float*
    bias, const float* norm, float* state, void* out, const lsh_seq_span_t* seqs, int n_seqs, const
    lsh_gla_shape_t* sh, lsh_stream_t stream);
int lsh_lm_gla_chunked_f32(const void* proj, int64_t ld, const float* low, const float* a2, const
    float* bias, const float* norm, float* state, void* out, float* workspace, const lsh_seq_span_t*
    seqs, int n_seqs, int max_n, int rows, const lsh_gla_shape_t* sh, lsh_stream_t stream);
int lsh_lm_gemm_epilogue_bf16(const void* A, int64_t lda, const void* W, void* C, int64_t ldc,
    float* C2, int64_t ld2, int n_split, int M, int N, int K, float scale, const float* bias,
    lsh_stream_t stream);
int lsh_lm_gemm_gated_bf16(const void* A, int64_t lda, const void* W, void* C, int64_t ldc, int M,
    int N, int K, int act, lsh_stream_t stream); /* act 0: silu, 1: relu */
int lsh_lm_residual_bf16(float* x, const lsh_residual_t* what, void* h, int rows, int width, float eps,
    const int* ids, const void* embed, int vocab, lsh_stream_t stream);
int lsh_lm_attn_decode_append_bf16(const void* proj, int64_t ld, int q_col, int k_col, void* k_cache,
    void* out, const int* row_slot, const int* row_pos, int rows, int max_len, float* workspace, const
    lsh_attn_shape_t* sh, const lsh_attn_mask_t* mask, lsh_stream_t stream);
int lsh_lm_gemm_planes2_bf16(const void* A0, int64_t lda0, const void* W0, float* C0, int K0, const
    void* A1, int64_t lda1, const void* W1, float* C1, int K1, int M, int N, int max_planes, int*
    planes0, int* planes1, lsh_stream_t stream);
int lsh_lm_gla_step_bf16(const void* proj, int64_t ld, const float* low, const float* a2, const float*
    bias, const float* norm, float* state, void* out, const int* row_slot, const int* row_pos, int
    rows, const lsh_gla_shape_t* sh, lsh_stream_t stream);
int lsh_lm_gla_scan_bf16(const void* proj, int64_t ld, const float* low, const float* a2, const float*
    bias, const float* norm, float* state, void* out, const lsh_seq_span_t* seqs, int n_seqs, const
    lsh_gla_shape_t* sh, lsh_stream_t stream);
int lsh_lm_gla_chunked_bf16(const void* proj, int64_t ld, const float* low, const float* a2, const
    float* bias, const float* norm, float* state, void* out, float* workspace, const lsh_seq_span_t*
    seqs, int n_seqs, int max_n, int rows, const lsh_gla_shape_t* sh, lsh_stream_t stream);

#ifdef __cplusplus
}
#endif
#endif /* LIGHTSEQ_LM_H_ */
