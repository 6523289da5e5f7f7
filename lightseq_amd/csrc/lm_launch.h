// C++ launchers of the floating-point decoder kernels (bfloat16 / float32 activations, float32
// residual stream).  Every mechanism is a launcher of its own with its constants as arguments.
// T is bf16_t or float throughout; sequences of a batch are packed row after row, without padding.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

#include "float_device.h"
#include "ls_launch.h"

namespace lsh {

// One sequence of a step: rows [row0, row0 + n) of the packed batch are its positions
// [pos0, pos0 + n); `slot` is its place in the caches and states.
struct SeqSpan {
  int row0, n, pos0, slot;
};

// ---- matrix products (gemm_float.hip) ---------------------------------------------------------
// C[m, n] = sum_k A[m, k] W[n, k].  Columns from n_split on go to the float matrix C2 (column
// n - n_split); n_split = N: none.  `planes` > 1 asks for that many partial sums over K, stored as
// float planes [planes][M][N] that the caller adds (few rows only; *planes_used says how many).
// The epilogue gives scale * sum + bias[n] (in float, before the result is rounded).
struct GemmEpilogue {
  float scale = 1.f;
  const float* bias = nullptr;  // [N]
};
template <typename T, typename TO>
int gemm_float(const T* A, long lda, const T* W, TO* C, long ldc, float* C2, long ld2, int n_split,
               int M, int N, int K, hipStream_t s, const GemmEpilogue& epilogue = GemmEpilogue());
template <typename T>
int gemm_float_planes(const T* A, long lda, const T* W, float* C, int M, int N, int K,
                      int max_planes, int* planes_used, hipStream_t s);
int gemm_float_preferred_planes(int M, int N, int K);
// two such products of different inputs and weights, in one launch for few rows
template <typename T>
struct FloatProduct {
  const T* A;
  long lda;
  const T* W;
  float* C;
  int K;
};
template <typename T>
int gemm_float_planes2(const FloatProduct<T>& p0, const FloatProduct<T>& p1, int M, int N,
                       int max_planes, int* planes0, int* planes1, hipStream_t s);

// C[m, n] = act(gate_n A[m]) * (up_n A[m]), weights [2][N][K]: the gates' rows, then the others
enum GateAct { kGateSilu = 0, kGateRelu = 1 };
template <typename T>
int gemm_gated(const T* A, long lda, const T* W, T* C, long ldc, int M, int N, int K, int act,
               hipStream_t s);

// Products over the rows that chose an expert.  A row is a (token, choice) pair, numbered
// token * top + choice; expert e serves rows list[e * tokens + 0 .. count[e]).
//  up:   act[row] = silu(gate_e h[token]) * (up_e h[token]), weights [experts][2][ff][width]
//  down: out[row] = down_e act[row],                         weights [experts][width][ff]
template <typename T>
int moe_up(const T* h, const T* w, T* act, const int* count, const int* list, int tokens, int top,
           int experts, int width, int ff, hipStream_t s);
template <typename T, typename TO>
int moe_down(const T* act, const T* w, TO* out, const int* count, const int* list, int tokens,
             int top, int experts, int width, int ff, hipStream_t s);

// ---- routing (moe_kernels.hip) ----------------------------------------------------------------
// The `top` largest of logits[token] + bias (the lower index first among equals) and the soft-max
// over them; fills the lists above.  count must be zero before (lm_norm's zero_count does it).
int moe_route(const float* logits, const float* bias, float* weight, int* count, int* list,
              int tokens, int experts, int top, hipStream_t s);
// the logits' product (float32 sums of h and w as they are) and the same choice, for few tokens
template <typename T>
int moe_router(const T* h, const T* w, const float* bias, float* weight, int* count, int* list,
               int tokens, int width, int experts, int top, hipStream_t s);

// ---- norms on the residual stream (lm_norm_kernels.hip) ---------------------------------------
enum NormKind {
  kLayerNorm = 0,  // (x - mean) / deviation * w + b
  kRmsNorm = 1,    // x / root mean square * w
};
// A summand of the residual row: parts many pieces, piece p of row r at
// y + p * part_stride + r * row_stride, times weight[r * parts + p] when weights are given.
struct AddPart {
  const void* y = nullptr;
  int parts = 0;
  long part_stride = 0, row_stride = 0;
  const float* weight = nullptr;
  const float *post_w = nullptr, *post_b = nullptr;  // norm of the sum of the pieces; null: none
};
// What is added before the norm: scale * (this summand + the second one).
struct AddSpec : AddPart {
  bool y_is_float = true;  // else T
  AddPart second;          // parts == 0: none
  float scale = 1.f;
  NormKind post_kind = kLayerNorm;
};
struct NormSpec {
  const float *w = nullptr, *b = nullptr;  // norm of the new residual row; w null: no output
  NormKind kind = kLayerNorm;
};
// Added to the row after that, ahead of the norm: its embedding again and / or a vector.
struct InjectSpec {
  const int* ids = nullptr;
  const float* vec = nullptr;  // [width]
  __host__ __device__ bool any() const { return ids || vec; }
};
// x[r] (+)= add; x[r] (+)= inject; h[r] = norm(x[r]).  With `ids`, x[r] = embed[ids[r]] to begin with.
// With `rows`, output row i comes from residual row rows[i] (no addition then).
// zero_count: n_zero ints set to zero for the routing that follows.
template <typename T>
int lm_norm(float* x, const AddSpec& add, const NormSpec& norm, T* h, int rows_n, int width,
            float eps, const int* ids, const T* embed, int vocab, const int* rows, int* zero_count,
            int n_zero, hipStream_t s, const InjectSpec& inject = InjectSpec());

// ---- attention (lm_attn_kernels.hip) ----------------------------------------------------------
struct AttnShape {
  int heads, kv_heads, dim, vdim;
  int dim_pad, vdim_pad;  // row lengths of the caches (attn_pad of dim and vdim)
  int max_step;           // positions per slot
};
int attn_pad(int dim);  // 0: not supported
// Per-head RMS norm (q and, unless shared, k), interleaved rotation with the table
// cos_sin[position][rot_pairs] of float2 (null: none), then q -> q_out[row][heads][dim_pad] and
// k, v -> slot caches [slot][kv_head][position][pad].  k_col < 0: the layer has no keys of its own;
// v_col < 0: its values are the keys.  Without norm weights there is no norm.
template <typename T>
int attn_prepare(const T* proj, long ld, int q_col, int k_col, int v_col, const float* q_norm,
                 const float* k_norm, float eps, const float2* cos_sin, int rot_pairs, T* q_out,
                 T* k_cache, T* v_cache, const int* row_slot, const int* row_pos, int rows,
                 const AttnShape& sh, hipStream_t s);
// Position i sees j <= i with i - j < window or j < keep_first (window <= 0: all), and with a chunk
// size only keys of its own chunk of positions (or kept ones).  sink: exp(sinks[head]) is added to
// the soft-max denominator, 1 without sinks.  v_cache == k_cache: the values are the keys.  out[row][heads * vdim] = context * sigmoid(gate) (gate: T
// columns of `proj` from g_col on; g_col < 0: none).
struct AttnMask {
  int window, keep_first;
  float scale;
  bool sink;
  int chunk = 0;                 // 0: none
  const float* sinks = nullptr;  // [heads]
  // the first position that `pos` sees beside the kept ones
  __host__ __device__ int first_seen(int pos) const {
    int lo = window > 0 && pos >= window ? pos - window + 1 : 0;
    if (chunk > 0) {
      const int c = pos - pos % chunk;
      lo = lo > c ? lo : c;
    }
    return lo;
  }
};
template <typename T>
int attn_prefill(const T* q, const T* k_cache, const T* v_cache, const T* proj, long ld, int g_col,
                 T* out, const SeqSpan* seqs, int n_seqs, int max_n, const AttnShape& sh,
                 const AttnMask& mask, hipStream_t s);
// one query row per sequence, row r at position row_pos[r] of slot row_slot[r].  max_len: no
// row_pos is >= max_len; workspace: attn_decode_workspace floats.
template <typename T>
int attn_decode(const T* q, const T* k_cache, const T* v_cache, const T* proj, long ld, int g_col,
                T* out, const int* row_slot, const int* row_pos, int rows, int max_len,
                float* workspace, const AttnShape& sh, const AttnMask& mask, hipStream_t s);
// The same with queries and the position's key straight from the projection, where the values are the
// keys: the key is appended to the cache on the way.
template <typename T>
int attn_decode_append(const T* proj, long ld, int q_col, int k_col, T* k_cache, T* out,
                       const int* row_slot, const int* row_pos, int rows, int max_len,
                       float* workspace, const AttnShape& sh, const AttnMask& mask, hipStream_t s);
bool attn_decode_append_supported(const AttnShape& sh, int q_col, int k_col, long ld);
size_t attn_decode_workspace(int rows, const AttnShape& sh);

// ---- gated delta rule (delta_kernels.hip) -----------------------------------------------------
struct DeltaShape {
  int heads, kv_heads, dim, vdim, taps;
  __host__ __device__ int channels() const { return 2 * kv_heads * dim + heads * vdim; }
};
// proj rows: [q | k | v | gate] columns, ba rows: [b (heads) | a (heads)] in float.
// conv_w [channels][taps]; conv_ring [slot][taps][channels] holds the inputs of the last taps
// positions, position p at p % taps; state [slot][heads][dim][vdim] in float.
// Short convolution + silu, unit q (times dim^-1/2) and k, log decay and beta of every row; the
// ring is brought up to the last position.
template <typename T>
int delta_prepare(const T* proj, long ld, const float* ba, const float* conv_w, const float* a_log,
                  const float* dt_bias, T* conv_ring, float* q, float* k, T* v, float* log_g,
                  float* beta, const SeqSpan* seqs, int n_seqs, int max_n, const DeltaShape& sh,
                  hipStream_t s);
// the recurrence over whole spans: token by token / in chunks of 64 on the matrix cores
template <typename T>
int delta_scan(const float* q, const float* k, const T* v, const float* log_g, const float* beta,
               float* state, float* o, const SeqSpan* seqs, int n_seqs, const DeltaShape& sh,
               hipStream_t s);
template <typename T>
int delta_chunked(const float* q, const float* k, const T* v, const float* log_g,
                  const float* beta, float* state, float* o, float* workspace,
                  const SeqSpan* seqs, int n_seqs, int max_n, int rows, const DeltaShape& sh,
                  hipStream_t s);
size_t delta_chunked_workspace(int rows, int n_seqs, const DeltaShape& sh);  // floats
bool delta_chunked_supported(const DeltaShape& sh);
// out = o / rms(o) * norm_w * silu(gate)
template <typename T>
int delta_gated_norm(const float* o, const T* proj, long ld, int g_col, const float* norm_w,
                     float eps, T* out, int rows, const DeltaShape& sh, hipStream_t s);
// one token per sequence, everything above in one launch
template <typename T>
int delta_step(const T* proj, long ld, int g_col, const float* ba, const float* conv_w,
               const float* a_log, const float* dt_bias, const float* norm_w, float eps,
               T* conv_ring, float* state, T* out, const int* row_slot, const int* row_pos,
               int rows, const DeltaShape& sh, hipStream_t s);

// ---- gated linear attention (gla_kernels.hip) ---------------------------------------------------
//   S <- diag(a) S + k v^T;  o = S^T (q dim^-1/2)  per head, a = sigmoid(A2 low + bias)^(1 / tau),
//   out = o / rms(o) * norm_w * silu(gate)
// proj rows hold q, k [heads][dim] and v, gate [heads][vdim] from the given columns on; `low` is the
// narrow product that the decay is made from, float [rows][rank] (rank: a multiple of 16, zero-padded);
// a2 [heads * dim][rank].  state [slot][heads][vdim][dim] in float.
struct GlaShape {
  int heads, dim, vdim, rank;
  int q_col, k_col, v_col, g_col;
  float inv_tau, eps;
};
struct GlaWeights {
  const float *a2, *bias, *norm;
};
// one token per sequence, row r at position row_pos[r] of slot row_slot[r]
template <typename T>
int gla_step(const T* proj, long ld, const float* low, const GlaWeights& w, float* state, T* out,
             const int* row_slot, const int* row_pos, int rows, const GlaShape& sh, hipStream_t s);
// whole spans: token by token / in chunks of 64 on the matrix cores
template <typename T>
int gla_scan(const T* proj, long ld, const float* low, const GlaWeights& w, float* state, T* out,
             const SeqSpan* seqs, int n_seqs, const GlaShape& sh, hipStream_t s);
template <typename T>
int gla_chunked(const T* proj, long ld, const float* low, const GlaWeights& w, float* state, T* out,
                float* workspace, const SeqSpan* seqs, int n_seqs, int max_n, int rows,
                const GlaShape& sh, hipStream_t s);
size_t gla_chunked_workspace(int rows, int n_seqs, const GlaShape& sh);  // floats
bool gla_chunked_supported(const GlaShape& sh, long ld);

// ---- sampling from float logits (lm_sample_kernels.hip) ---------------------------------------
// Chooses a token per row (greedy: topk == 1; topk > 1; or topp in (0, 1] with topk == 0), writes
// it to ids[row * max_step + row_len[row]] and last_ids[row], advances row_len and row_pos; a row
// that has ended (its last id is eos) repeats eos without advancing its text.  unfinished is set
// to 1 by every row whose new token is not eos.
int lm_sample(const float* logits, int rows, int vocab, int topk, float topp, int eos_id,
              void* rng_state, int* ids, int max_step, int* last_ids, int* row_len, int* row_pos,
              int* unfinished, hipStream_t s);

}  // namespace lsh
