// extern "C" surface of the floating-point decoder kernels (include/lightseq_lm.h).
#include "../../include/lightseq_lm.h"

#include "lm_launch.h"

using namespace lsh;

#define HS(s) reinterpret_cast<hipStream_t>(s)

namespace {

AttnShape shape_of(const lsh_attn_shape_t& a) {
  return AttnShape{a.heads, a.kv_heads, a.dim, a.vdim, attn_pad(a.dim), attn_pad(a.vdim), a.max_step};
}
AttnMask mask_of(const lsh_attn_mask_t& m) {
  return AttnMask{m.window, m.keep_first, m.scale, m.sink != 0, m.chunk, m.sinks};
}
GlaShape shape_of(const lsh_gla_shape_t& g) {
  return GlaShape{g.heads, g.dim, g.vdim, g.rank, g.q_col, g.k_col, g.v_col, g.g_col,
                  1.f / g.tau, g.eps};
}
void part_of(const lsh_residual_part_t& p, AddPart& out) {
  if (!p.y) return;
  out = AddPart{p.y, p.parts, (long)p.part_stride, (long)p.row_stride, p.weight, p.post_w, p.post_b};
}
DeltaShape shape_of(const lsh_delta_shape_t& d) {
  return DeltaShape{d.heads, d.kv_heads, d.dim, d.vdim, d.taps};
}
static_assert(sizeof(lsh_seq_span_t) == sizeof(SeqSpan), "the same four ints");
const SeqSpan* spans(const lsh_seq_span_t* s) { return reinterpret_cast<const SeqSpan*>(s); }

#define NEED(p) \
  if (!(p)) return lsh_fail(LSH_ERR_INVALID, "null descriptor")

}  // namespace

extern "C" {

int lsh_lm_attn_pad(int dim) { return attn_pad(dim); }
int64_t lsh_lm_attn_decode_workspace(int rows, const lsh_attn_shape_t* sh) {
  return sh ? (int64_t)attn_decode_workspace(rows, shape_of(*sh)) : 0;
}
int64_t lsh_lm_delta_chunked_workspace(int rows, int n_seqs, const lsh_delta_shape_t* sh) {
  return sh ? (int64_t)delta_chunked_workspace(rows, n_seqs, shape_of(*sh)) : 0;
}
int lsh_lm_delta_chunked_supported(const lsh_delta_shape_t* sh) {
  return sh && delta_chunked_supported(shape_of(*sh)) ? 1 : 0;
}

int64_t lsh_lm_gla_chunked_workspace(int rows, int n_seqs, const lsh_gla_shape_t* sh) {
  return sh ? (int64_t)gla_chunked_workspace(rows, n_seqs, shape_of(*sh)) : 0;
}
int lsh_lm_gla_chunked_supported(const lsh_gla_shape_t* sh, int64_t ld) {
  return sh && gla_chunked_supported(shape_of(*sh), ld) ? 1 : 0;
}

int lsh_lm_moe_route(const float* logits, const float* bias, float* weight, int* count, int* list,
                     int tokens, int experts, int top, lsh_stream_t s) {
  return moe_route(logits, bias, weight, count, list, tokens, experts, top, HS(s));
}

int lsh_lm_sample(const float* logits, int rows, int vocab, int topk, float topp, int eos_id,
                  void* rng_state, int* ids, int max_step, int* last_ids, int* row_len, int* row_pos,
                  int* unfinished, lsh_stream_t s) {
  return lm_sample(logits, rows, vocab, topk, topp, eos_id, rng_state, ids, max_step, last_ids,
                   row_len, row_pos, unfinished, HS(s));
}

#define LM_TYPED(SUF, T)                                                                           \
  int lsh_lm_gemm_##SUF(const void* A, int64_t lda, const void* W, void* C, int64_t ldc,       \
                        float* C2, int64_t ld2, int n_split, int M, int N, int K,                \
                        lsh_stream_t s) {                                                          \
    return gemm_float<T, T>((const T*)A, lda, (const T*)W, (T*)C, ldc, C2, ld2, n_split, M, N, K,  \
                            HS(s));                                                                \
  }                                                                                                \
  int lsh_lm_gemm_f32_out_##SUF(const void* A, int64_t lda, const void* W, float* C, int M,      \
                                int N, int K, lsh_stream_t s) {                                    \
    return gemm_float<T, float>((const T*)A, lda, (const T*)W, C, N, nullptr, 0, N, M, N, K,       \
                                HS(s));                                                            \
  }                                                                                                \
  int lsh_lm_gemm_planes_##SUF(const void* A, int64_t lda, const void* W, float* C, int M,       \
                               int N, int K, int max_planes, int* planes_used, lsh_stream_t s) {   \
    NEED(planes_used);                                                                             \
    return gemm_float_planes<T>((const T*)A, lda, (const T*)W, C, M, N, K, max_planes,             \
                                planes_used, HS(s));                                               \
  }                                                                                                \
  int lsh_lm_moe_router_##SUF(const void* h, const void* w, const float* bias, float* weight,       \
                              int* count, int* list, int tokens, int width, int experts, int top,  \
                              lsh_stream_t s) {                                                    \
    return moe_router<T>((const T*)h, (const T*)w, bias, weight, count, list, tokens, width,       \
                         experts, top, HS(s));                                                     \
  }                                                                                                \
  int lsh_lm_moe_up_##SUF(const void* h, const void* w, void* act, const int* count,               \
                          const int* list, int tokens, int top, int experts, int width, int ff,    \
                          lsh_stream_t s) {                                                        \
    return moe_up<T>((const T*)h, (const T*)w, (T*)act, count, list, tokens, top, experts, width,  \
                     ff, HS(s));                                                                   \
  }                                                                                                \
  int lsh_lm_moe_down_##SUF(const void* act, const void* w, void* out, const int* count,           \
                            const int* list, int tokens, int top, int experts, int width, int ff,  \
                            lsh_stream_t s) {                                                      \
    return moe_down<T, T>((const T*)act, (const T*)w, (T*)out, count, list, tokens, top, experts,  \
                          width, ff, HS(s));                                                       \
  }                                                                                                \
  int lsh_lm_norm_##SUF(float* x, const void* y, int y_is_float, int parts, int64_t part_stride, \
                        int64_t row_stride, const float* weight, const float* post_w,            \
                        const float* post_b, const float* norm_w, const float* norm_b, void* h,    \
                        int rows, int width, float eps, const int* ids, const void* embed,         \
                        int vocab, const int* from_rows, int* zero_count, int n_zero,              \
                        lsh_stream_t s) {                                                          \
    AddSpec add;                                                                                   \
    add.y = y;                                                                                     \
    add.y_is_float = y_is_float != 0;                                                              \
    add.parts = parts;                                                                             \
    add.part_stride = part_stride;                                                                 \
    add.row_stride = row_stride;                                                                   \
    add.weight = weight;                                                                           \
    add.post_w = post_w;                                                                           \
    add.post_b = post_b;                                                                           \
    return lm_norm<T>(x, add, NormSpec{norm_w, norm_b}, (T*)h, rows, width, eps, ids,              \
                      (const T*)embed, vocab, from_rows, zero_count, n_zero, HS(s));               \
  }                                                                                                \
  int lsh_lm_attn_prepare_##SUF(const void* proj, int64_t ld, int q_col, int k_col, int v_col,   \
                                const float* q_norm, const float* k_norm, float eps,               \
                                const float* cos_sin, int rot_pairs, void* q_out, void* k_cache,   \
                                void* v_cache, const int* row_slot, const int* row_pos, int rows,  \
                                const lsh_attn_shape_t* sh, lsh_stream_t s) {                      \
    NEED(sh);                                                                                      \
    return attn_prepare<T>((const T*)proj, ld, q_col, k_col, v_col, q_norm, k_norm, eps,           \
                           (const float2*)cos_sin, rot_pairs, (T*)q_out, (T*)k_cache, (T*)v_cache, \
                           row_slot, row_pos, rows, shape_of(*sh), HS(s));                         \
  }                                                                                                \
  int lsh_lm_attn_prefill_##SUF(const void* q, const void* k_cache, const void* v_cache,           \
                                const void* proj, int64_t ld, int g_col, void* out,              \
                                const lsh_seq_span_t* seqs, int n_seqs, int max_n,                 \
                                const lsh_attn_shape_t* sh, const lsh_attn_mask_t* mask,           \
                                lsh_stream_t s) {                                                  \
    NEED(sh && mask);                                                                              \
    return attn_prefill<T>((const T*)q, (const T*)k_cache, (const T*)v_cache, (const T*)proj, ld,  \
                           g_col, (T*)out, spans(seqs), n_seqs, max_n, shape_of(*sh),              \
                           mask_of(*mask), HS(s));                                                 \
  }                                                                                                \
  int lsh_lm_attn_decode_##SUF(const void* q, const void* k_cache, const void* v_cache,            \
                               const void* proj, int64_t ld, int g_col, void* out,               \
                               const int* row_slot, const int* row_pos, int rows, int max_len,     \
                               float* workspace, const lsh_attn_shape_t* sh,                       \
                               const lsh_attn_mask_t* mask, lsh_stream_t s) {                      \
    NEED(sh && mask);                                                                              \
    return attn_decode<T>((const T*)q, (const T*)k_cache, (const T*)v_cache, (const T*)proj, ld,   \
                          g_col, (T*)out, row_slot, row_pos, rows, max_len, workspace,             \
                          shape_of(*sh), mask_of(*mask), HS(s));                                   \
  }                                                                                                \
  int lsh_lm_delta_prepare_##SUF(const void* proj, int64_t ld, const float* ba,                  \
                                 const float* conv_w, const float* a_log, const float* dt_bias,    \
                                 void* conv_ring, float* q, float* k, void* v, float* log_g,       \
                                 float* beta, const lsh_seq_span_t* seqs, int n_seqs, int max_n,   \
                                 const lsh_delta_shape_t* sh, lsh_stream_t s) {                    \
    NEED(sh);                                                                                      \
    return delta_prepare<T>((const T*)proj, ld, ba, conv_w, a_log, dt_bias, (T*)conv_ring, q, k,   \
                            (T*)v, log_g, beta, spans(seqs), n_seqs, max_n, shape_of(*sh), HS(s)); \
  }                                                                                                \
  int lsh_lm_delta_scan_##SUF(const float* q, const float* k, const void* v, const float* log_g,   \
                              const float* beta, float* state, float* o,                           \
                              const lsh_seq_span_t* seqs, int n_seqs, const lsh_delta_shape_t* sh, \
                              lsh_stream_t s) {                                                    \
    NEED(sh);                                                                                      \
    return delta_scan<T>(q, k, (const T*)v, log_g, beta, state, o, spans(seqs), n_seqs,            \
                         shape_of(*sh), HS(s));                                                    \
  }                                                                                                \
  int lsh_lm_delta_chunked_##SUF(const float* q, const float* k, const void* v,                    \
                                 const float* log_g, const float* beta, float* state, float* o,    \
                                 float* workspace, const lsh_seq_span_t* seqs, int n_seqs,         \
                                 int max_n, int rows, const lsh_delta_shape_t* sh,                 \
                                 lsh_stream_t s) {                                                 \
    NEED(sh);                                                                                      \
    return delta_chunked<T>(q, k, (const T*)v, log_g, beta, state, o, workspace, spans(seqs),      \
                            n_seqs, max_n, rows, shape_of(*sh), HS(s));                            \
  }                                                                                                \
  int lsh_lm_delta_gated_norm_##SUF(const float* o, const void* proj, int64_t ld, int g_col,     \
                                    const float* norm_w, float eps, void* out, int rows,           \
                                    const lsh_delta_shape_t* sh, lsh_stream_t s) {                 \
    NEED(sh);                                                                                      \
    return delta_gated_norm<T>(o, (const T*)proj, ld, g_col, norm_w, eps, (T*)out, rows,           \
                               shape_of(*sh), HS(s));                                              \
  }                                                                                                \
  int lsh_lm_delta_step_##SUF(const void* proj, int64_t ld, int g_col, const float* ba,          \
                              const float* conv_w, const float* a_log, const float* dt_bias,       \
                              const float* norm_w, float eps, void* conv_ring, float* state,       \
                              void* out, const int* row_slot, const int* row_pos, int rows,        \
                              const lsh_delta_shape_t* sh, lsh_stream_t s) {                       \
    NEED(sh);                                                                                      \
    return delta_step<T>((const T*)proj, ld, g_col, ba, conv_w, a_log, dt_bias, norm_w, eps,       \
                         (T*)conv_ring, state, (T*)out, row_slot, row_pos, rows, shape_of(*sh),    \
                         HS(s));                                                                   \
  } \
  int lsh_lm_gemm_epilogue_##SUF(const void* A, int64_t lda, const void* W, void* C, int64_t ldc,  \
                                 float* C2, int64_t ld2, int n_split, int M, int N, int K,         \
                                 float scale, const float* bias, lsh_stream_t s) {                 \
    GemmEpilogue e;                                                                                \
    e.scale = scale;                                                                               \
    e.bias = bias;                                                                                 \
    return gemm_float<T, T>((const T*)A, lda, (const T*)W, (T*)C, ldc, C2, ld2, n_split, M, N, K,  \
                            HS(s), e);                                                             \
  }                                                                                                \
  int lsh_lm_gemm_gated_##SUF(const void* A, int64_t lda, const void* W, void* C, int64_t ldc,     \
                              int M, int N, int K, int act, lsh_stream_t s) {                      \
    return gemm_gated<T>((const T*)A, lda, (const T*)W, (T*)C, ldc, M, N, K, act, HS(s));          \
  }                                                                                                \
  int lsh_lm_residual_##SUF(float* x, const lsh_residual_t* what, void* h, int rows, int width,    \
                            float eps, const int* ids, const void* embed, int vocab,               \
                            lsh_stream_t s) {                                                      \
    NEED(what);                                                                                    \
    AddSpec add;                                                                                   \
    part_of(what->part[0], add);                                                                   \
    part_of(what->part[1], add.second);                                                            \
    add.y_is_float = what->y_is_float != 0;                                                        \
    add.scale = what->scale;                                                                       \
    add.post_kind = what->post_rms ? kRmsNorm : kLayerNorm;                                        \
    const NormSpec norm{what->norm_w, what->norm_b, what->norm_rms ? kRmsNorm : kLayerNorm};       \
    const InjectSpec inject{what->inject_ids, what->inject_vec};                                   \
    return lm_norm<T>(x, add, norm, (T*)h, rows, width, eps, ids, (const T*)embed, vocab, nullptr, \
                      nullptr, 0, HS(s), inject);                                                  \
  }                                                                                                \
  int lsh_lm_attn_decode_append_##SUF(const void* proj, int64_t ld, int q_col, int k_col,          \
                                      void* k_cache, void* out, const int* row_slot,               \
                                      const int* row_pos, int rows, int max_len, float* workspace, \
                                      const lsh_attn_shape_t* sh, const lsh_attn_mask_t* mask,     \
                                      lsh_stream_t s) {                                            \
    NEED(sh && mask);                                                                              \
    return attn_decode_append<T>((const T*)proj, ld, q_col, k_col, (T*)k_cache, (T*)out, row_slot, \
                                 row_pos, rows, max_len, workspace, shape_of(*sh), mask_of(*mask), \
                                 HS(s));                                                           \
  }                                                                                                \
  int lsh_lm_gemm_planes2_##SUF(const void* A0, int64_t lda0, const void* W0, float* C0, int K0,   \
                                const void* A1, int64_t lda1, const void* W1, float* C1, int K1,   \
                                int M, int N, int max_planes, int* planes0, int* planes1,          \
                                lsh_stream_t s) {                                                  \
    NEED(planes0 && planes1);                                                                      \
    return gemm_float_planes2<T>(FloatProduct<T>{(const T*)A0, lda0, (const T*)W0, C0, K0},        \
                                 FloatProduct<T>{(const T*)A1, lda1, (const T*)W1, C1, K1}, M, N,  \
                                 max_planes, planes0, planes1, HS(s));                             \
  }                                                                                                \
  int lsh_lm_gla_step_##SUF(const void* proj, int64_t ld, const float* low, const float* a2,       \
                            const float* bias, const float* norm, float* state, void* out,         \
                            const int* row_slot, const int* row_pos, int rows,                     \
                            const lsh_gla_shape_t* sh, lsh_stream_t s) {                           \
    NEED(sh);                                                                                      \
    return gla_step<T>((const T*)proj, ld, low, GlaWeights{a2, bias, norm}, state, (T*)out,        \
                       row_slot, row_pos, rows, shape_of(*sh), HS(s));                             \
  }                                                                                                \
  int lsh_lm_gla_scan_##SUF(const void* proj, int64_t ld, const float* low, const float* a2,       \
                            const float* bias, const float* norm, float* state, void* out,         \
                            const lsh_seq_span_t* seqs, int n_seqs, const lsh_gla_shape_t* sh,     \
                            lsh_stream_t s) {                                                      \
    NEED(sh);                                                                                      \
    return gla_scan<T>((const T*)proj, ld, low, GlaWeights{a2, bias, norm}, state, (T*)out,        \
                       spans(seqs), n_seqs, shape_of(*sh), HS(s));                                 \
  }                                                                                                \
  int lsh_lm_gla_chunked_##SUF(const void* proj, int64_t ld, const float* low, const float* a2,    \
                               const float* bias, const float* norm, float* state, void* out,      \
                               float* workspace, const lsh_seq_span_t* seqs, int n_seqs, int max_n,\
                               int rows, const lsh_gla_shape_t* sh, lsh_stream_t s) {              \
    NEED(sh);                                                                                      \
    return gla_chunked<T>((const T*)proj, ld, low, GlaWeights{a2, bias, norm}, state, (T*)out,     \
                          workspace, spans(seqs), n_seqs, max_n, rows, shape_of(*sh), HS(s));      \
  }

LM_TYPED(f32, float)
LM_TYPED(bf16, bf16_t)

}  // extern "C"
