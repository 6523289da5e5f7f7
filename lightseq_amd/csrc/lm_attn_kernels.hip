// Attention of the floating-point decoders over slot caches [slot][kv_head][position][pad]: per-head
// RMS norm and interleaved rotation, causal attention with a sliding window, kept first tokens and
// a valueless sink in the soft-max, and an element-wise output gate; a prompt kernel on the matrix
// cores and a one-token kernel that streams the cache.
//
// Keys and values are stored with rows padded to a size the prompt kernel is instantiated for
// (attn_pad), the padding written as zeros with the row, so no load needs a column guard.
#include <algorithm>

#include "lm_launch.h"

namespace lsh {

int attn_pad(int dim) {
  return dim <= 0 ? 0 : dim <= 64 ? 64 : dim <= 96 ? 96 : dim <= 128 ? 128 : dim <= 256 ? 256 : 0;
}

namespace {

// ------------------------------------------------------------------------------------------------
// One wavefront per (row, head); lane i holds the pairs i, i + 64 (dimensions 2i, 2i + 1).
template <typename T>
__global__ void __launch_bounds__(256)
attn_prepare_kernel(const T* __restrict__ proj, long ld, int q_col, int k_col, int v_col,
                    const float* __restrict__ q_norm, const float* __restrict__ k_norm, float eps,
                    const float2* __restrict__ cos_sin, int rot_pairs, T* __restrict__ q_out,
                    T* __restrict__ k_cache, T* __restrict__ v_cache,
                    const int* __restrict__ row_slot, const int* __restrict__ row_pos, long units,
                    int heads_per_row, AttnShape sh) {
  const long unit = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (unit >= units) return;
  const int lane = threadIdx.x & 63;
  const long row = unit / heads_per_row;
  int head = (int)(unit - row * heads_per_row);
  const T* src = proj + row * ld;
  const int pos = row_pos[row];
  int kind = 0;  // 0 q, 1 k, 2 v
  T* dst;
  if (head < sh.heads) {
    src += q_col + head * sh.dim;
    dst = q_out + (row * sh.heads + head) * sh.dim_pad;
  } else {
    head -= sh.heads;
    kind = head < sh.kv_heads ? 1 : 2;
    if (kind == 2) head -= sh.kv_heads;
    src += kind == 1 ? k_col + head * sh.dim : v_col + head * sh.vdim;
    const long at = ((long)row_slot[row] * sh.kv_heads + head) * sh.max_step + pos;
    dst = kind == 1 ? k_cache + at * sh.dim_pad : v_cache + at * sh.vdim_pad;
  }
  const int n = kind == 2 ? sh.vdim : sh.dim, pad = kind == 2 ? sh.vdim_pad : sh.dim_pad;
  float u[2][2];
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int d = 2 * (i * 64 + lane);
    u[i][0] = d < n ? to_f(src[d]) : 0.f;
    u[i][1] = d + 1 < n ? to_f(src[d + 1]) : 0.f;
  }
  if (kind != 2) {
    const float ss = wave_sum_dpp(u[0][0] * u[0][0] + u[0][1] * u[0][1] + u[1][0] * u[1][0] +
                                  u[1][1] * u[1][1]);
    const float r = 1.0f / sqrtf(ss / (float)n + eps);
    const float* w = kind == 0 ? q_norm : k_norm;
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int p = i * 64 + lane, d = 2 * p;
      if (w) {
        if (d < n) u[i][0] = u[i][0] * r * w[d];
        if (d + 1 < n) u[i][1] = u[i][1] * r * w[d + 1];
      }
      if (p < rot_pairs) {
        const float2 cs = cos_sin[(long)pos * rot_pairs + p];
        const float a = u[i][0], b = u[i][1];
        u[i][0] = a * cs.x - b * cs.y;
        u[i][1] = b * cs.x + a * cs.y;
      }
    }
  }
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int d = 2 * (i * 64 + lane);
    if (d < pad) stv<2, T>(dst + d, u[i]);  // zeros beyond the head size
  }
}

// The same for head sizes, columns and row lengths in fours: LPH lanes per head, four elements (two
// pairs) per lane, 64 / LPH heads per wavefront.
template <typename T, int LPH>
__global__ void __launch_bounds__(256)
attn_prepare4_kernel(const T* __restrict__ proj, long ld, int q_col, int k_col, int v_col,
                     const float* __restrict__ q_norm, const float* __restrict__ k_norm, float eps,
                     const float2* __restrict__ cos_sin, int rot_pairs, T* __restrict__ q_out,
                     T* __restrict__ k_cache, T* __restrict__ v_cache,
                     const int* __restrict__ row_slot, const int* __restrict__ row_pos, int units,
                     int heads_per_row, AttnShape sh) {
  const int unit_raw = (int)((blockIdx.x * 256 + threadIdx.x) / LPH);
  const int unit = min(unit_raw, units - 1);  // every lane takes part in the exchanges
  const int d = (threadIdx.x % LPH) * 4;
  const int row = unit / heads_per_row;
  int head = unit - row * heads_per_row;
  const int pos = row_pos[row];
  const T* src = proj + row * ld;
  int kind = 0;
  T* dst;
  if (head < sh.heads) {
    src += q_col + head * sh.dim;
    dst = q_out + ((long)row * sh.heads + head) * sh.dim_pad;
  } else {
    head -= sh.heads;
    kind = head < sh.kv_heads ? 1 : 2;
    if (kind == 2) head -= sh.kv_heads;
    src += kind == 1 ? k_col + head * sh.dim : v_col + head * sh.vdim;
    const long at = ((long)row_slot[row] * sh.kv_heads + head) * sh.max_step + pos;
    dst = kind == 1 ? k_cache + at * sh.dim_pad : v_cache + at * sh.vdim_pad;
  }
  const int n = kind == 2 ? sh.vdim : sh.dim, pad = kind == 2 ? sh.vdim_pad : sh.dim_pad;
  float u[4] = {0.f, 0.f, 0.f, 0.f};
  if (d < n) ldv<4, T>(src + d, u);
  float ss = u[0] * u[0] + u[1] * u[1] + u[2] * u[2] + u[3] * u[3];
  ss += dpp_f<kDppXor1>(ss);
  ss += dpp_f<kDppXor2>(ss);
  ss += dpp_f<kDppHalfMirror>(ss);
  ss += dpp_f<kDppMirror>(ss);
  if (LPH > 16) ss += __shfl_xor(ss, 16);
  if (LPH > 32) ss += __shfl_xor(ss, 32);
  if (kind != 2) {
    const float r = 1.0f / sqrtf(ss / (float)n + eps);
    const float* w = kind == 0 ? q_norm : k_norm;
    if (w && d < n) {
      float wv[4];
      ldv<4, float>(w + d, wv);
#pragma unroll
      for (int e = 0; e < 4; ++e) u[e] = u[e] * r * wv[e];
    }
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int p = d / 2 + i;
      if (p < rot_pairs) {
        const float2 cs = cos_sin[(long)pos * rot_pairs + p];
        const float a = u[2 * i], b = u[2 * i + 1];
        u[2 * i] = a * cs.x - b * cs.y;
        u[2 * i + 1] = b * cs.x + a * cs.y;
      }
    }
  }
  if (unit_raw < units && d < pad) stv<4, T>(dst + d, u);
}

// ------------------------------------------------------------------------------------------------
// Prompt kernel.  A workgroup takes 128 queries of one (sequence, head), 32 per wavefront, and walks
// the key tiles of 64 that any of them sees: first the kept tokens, then the window.  Scores are
// computed transposed (keys x queries), so a lane owns one query: running maximum, sum and the
// rescaling of its context need no exchange but one with the other half of the wavefront, and the
// probabilities are the second operand of the context product as they lie in registers.  The sink
// is the start value of the running soft-max: its logit as the maximum, sum 1, context 0.
constexpr int kQT = 128, kKT = 64;
constexpr float kLog2e = 1.44269504088896340736f;

__device__ __forceinline__ float exp2_f(float x) { return __builtin_amdgcn_exp2f(x); }

template <typename T, int NK, int NV>  // head sizes in 32s
__global__ void __launch_bounds__(256, sizeof(T) == 2 && NK <= 4 && NV <= 4 ? 2 : 1)
attn_prefill_kernel(const T* __restrict__ q, const T* __restrict__ k_cache,
                    const T* __restrict__ v_cache, const T* __restrict__ proj, long ld, int g_col,
                    T* __restrict__ out, const SeqSpan* __restrict__ seqs, AttnShape sh,
                    AttnMask mask) {
  constexpr int DP = NK * 32, VP = NV * 32, V = FT<T>::kVec;
  constexpr int KSTR = DP + V;           // elements per key row in LDS
  constexpr int VSTR = kKT + 16 / sizeof(T);  // keys per value column in LDS
  constexpr int NKS = DP * sizeof(T) / 32;    // 32-byte slices of a key row
  extern __shared__ __attribute__((aligned(16))) char smem_raw[];
  T* Ks = reinterpret_cast<T*>(smem_raw);
  T* Vt = Ks + kKT * KSTR;
  const SeqSpan sq = seqs[blockIdx.z];
  // the longest key ranges first
  const int qt = (sq.n + kQT - 1) / kQT - 1 - (int)blockIdx.x;
  if (qt < 0) return;
  const int head = blockIdx.y, kvh = head / (sh.heads / sh.kv_heads);
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l32 = lane & 31, g = lane >> 5;
  const int i0 = qt * kQT;                      // first query of the tile, in the span
  const int i_last = min(i0 + kQT, sq.n) - 1;
  const int my_i = min(i0 + wave * 32 + l32, sq.n - 1);
  const int pos = sq.pos0 + my_i;
  const int wq_lo = sq.pos0 + min(i0 + wave * 32, sq.n - 1);
  const int wq_hi = sq.pos0 + min(i0 + wave * 32 + 31, sq.n - 1);
  // first keys that the wavefront's first, last and this lane's query see (kept ones apart)
  const int lo_first = mask.first_seen(wq_lo), lo_last = mask.first_seen(wq_hi);
  const int lo_mine = mask.first_seen(pos);
  const bool wave_live = i0 + wave * 32 < sq.n;
  const int kv_len = sq.pos0 + sq.n;
  const long cache0 = ((long)sq.slot * sh.kv_heads + kvh) * sh.max_step;
  const T* kc = k_cache + cache0 * DP;
  const T* vc = v_cache + cache0 * VP;

  frag_t qf[NKS];
  {
    const T* qr = q + ((long)(sq.row0 + my_i) * sh.heads + head) * DP;
#pragma unroll
    for (int s = 0; s < NKS; ++s) qf[s] = *reinterpret_cast<const frag_t*>(qr + (2 * s + g) * V);
  }
  const float sc2 = mask.scale * kLog2e;
  // m in units of log2
  float m = !mask.sink ? -INFINITY : mask.sinks ? mask.sinks[head] * kLog2e : 0.f;
  float l = mask.sink ? 1.f : 0.f;
  f32x16v acc[NV];
#pragma unroll
  for (int d = 0; d < NV; ++d) acc[d] = (f32x16v)0.f;

  const int first_pos = sq.pos0 + i0, last_pos = sq.pos0 + i_last;
  const int t_end = last_pos / kKT;  // last tile
  const int t_win = mask.first_seen(first_pos) / kKT;
  const int t_keep = mask.keep_first > 0 ? (min(mask.keep_first, kv_len) - 1) / kKT : -1;
  // the next tile's keys (16-byte chunks; rows beyond the sequence are clamped, their scores are
  // masked) and values (4 keys x 4 columns per unit; rows beyond it are zero) wait in registers
  // while the present one is used
  typedef T T4 __attribute__((ext_vector_type(4)));
  constexpr int CH = DP / V, KU = kKT * CH / 256;
  constexpr int VU = ((kKT / 4) * (VP / 4) + 255) / 256;
  frag_t kr[KU];
  T4 vr[VU][4];
  auto fetch = [&](int key0) {
#pragma unroll
    for (int u = 0; u < KU; ++u) {
      const int c = u * 256 + tid, r = c / CH, x = c - r * CH;
      kr[u] = *reinterpret_cast<const frag_t*>(kc + (long)min(key0 + r, kv_len - 1) * DP + x * V);
    }
#pragma unroll
    for (int u = 0; u < VU; ++u) {
      const int c = u * 256 + tid, r4 = c / (VP / 4), x = c - r4 * (VP / 4);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int key = key0 + r4 * 4 + j;
        vr[u][j] = key < kv_len && r4 < kKT / 4 ? *reinterpret_cast<const T4*>(vc + (long)key * VP + x * 4)
                                                : (T4)0.f;
      }
    }
  };
  auto next_tile = [&](int t) {
    ++t;
    return t > t_keep && t < t_win ? t_win : t;
  };
  int t = next_tile(-1);
  fetch(t * kKT);
  for (; t <= t_end; t = next_tile(t)) {
    const int key0 = t * kKT;
    __syncthreads();
#pragma unroll
    for (int u = 0; u < KU; ++u) {
      const int c = u * 256 + tid, r = c / CH, x = c - r * CH;
      *reinterpret_cast<frag_t*>(&Ks[r * KSTR + x * V]) = kr[u];
    }
#pragma unroll
    for (int u = 0; u < VU; ++u) {
      const int c = u * 256 + tid, r4 = c / (VP / 4), x = c - r4 * (VP / 4);
      if (r4 < kKT / 4) {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const T4 col = {vr[u][0][e], vr[u][1][e], vr[u][2][e], vr[u][3][e]};
          *reinterpret_cast<T4*>(&Vt[(x * 4 + e) * VSTR + r4 * 4]) = col;
        }
      }
    }
    if (next_tile(t) <= t_end) fetch(next_tile(t) * kKT);
    __syncthreads();
    if (!wave_live) continue;
    // does any query of this wavefront see any key of the tile?
    const bool causal_any = key0 <= wq_hi;
    const bool win_any = key0 + kKT - 1 >= lo_first;
    if (!causal_any || !(win_any || key0 < mask.keep_first)) continue;
    const bool all = key0 + kKT - 1 <= wq_lo && (key0 >= lo_last || key0 + kKT <= mask.keep_first);
    f32x16v sc[2];
#pragma unroll
    for (int b = 0; b < 2; ++b) {
      sc[b] = (f32x16v)0.f;
      const T* kr = &Ks[(b * 32 + l32) * KSTR + g * V];
#pragma unroll
      for (int s = 0; s < NKS; ++s)
        sc[b] = mma32(T{}, *reinterpret_cast<const frag_t*>(kr + 2 * s * V), qf[s], sc[b]);
    }
    float mx = m;
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        float v = sc[b][i] * sc2;
        if (!all) {
          const int key = key0 + b * 32 + 8 * (i >> 2) + 4 * g + (i & 3);
          const bool see = key <= pos && (key >= lo_mine || key < mask.keep_first);
          v = see ? v : -INFINITY;
        }
        sc[b][i] = v;
        mx = fmaxf(mx, v);
      }
    mx = fmaxf(mx, __shfl_xor(mx, 32));
    const float f = m == -INFINITY ? 0.f : exp2_f(m - mx);
    m = mx;
    // (no sink) a query that has seen nothing yet: all its probabilities are zero
    const float ref = mx == -INFINITY ? 0.f : mx;
    float sum = 0.f;
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        sc[b][i] = exp2_f(sc[b][i] - ref);
        sum += sc[b][i];
      }
    sum += __shfl_xor(sum, 32);
    l = l * f + sum;
#pragma unroll
    for (int d = 0; d < NV; ++d)
#pragma unroll
      for (int i = 0; i < 16; ++i) acc[d][i] *= f;
    // context: slots of the product are the keys in the order the scores lie in registers
#pragma unroll
    for (int b = 0; b < 2; ++b) {
      if constexpr (sizeof(T) == 2) {
#pragma unroll
        for (int h = 0; h < 2; ++h) {
          bf16x8 pb;
#pragma unroll
          for (int j = 0; j < 8; ++j) pb[j] = (__bf16)sc[b][8 * h + j];
#pragma unroll
          for (int d = 0; d < NV; ++d) {
            const T* vr = &Vt[(d * 32 + l32) * VSTR + b * 32 + 16 * h + 4 * g];
            const uint2 lo = *reinterpret_cast<const uint2*>(vr);
            const uint2 hi = *reinterpret_cast<const uint2*>(vr + 8);
            const frag_t va = {lo.x, lo.y, hi.x, hi.y};
            acc[d] = mma32(T{}, va, __builtin_bit_cast(frag_t, pb), acc[d]);
          }
        }
      } else {
#pragma unroll
        for (int h = 0; h < 4; ++h) {
          const f32x4 pb = {sc[b][4 * h], sc[b][4 * h + 1], sc[b][4 * h + 2], sc[b][4 * h + 3]};
#pragma unroll
          for (int d = 0; d < NV; ++d) {
            const frag_t va = *reinterpret_cast<const frag_t*>(
                &Vt[(d * 32 + l32) * VSTR + b * 32 + 8 * h + 4 * g]);
            acc[d] = mma32(T{}, va, __builtin_bit_cast(frag_t, pb), acc[d]);
          }
        }
      }
    }
  }
  if (i0 + wave * 32 + l32 >= sq.n) return;
  const float inv = l > 0.f ? 1.f / l : 0.f;
  const long row = sq.row0 + my_i;
  const T* gate = g_col >= 0 ? proj + row * ld + g_col + head * sh.vdim : nullptr;
  T* op = out + row * ((long)sh.heads * sh.vdim) + head * sh.vdim;
  const bool vec = sh.vdim % 4 == 0 && (g_col < 0 || (g_col % 4 == 0 && ld % 4 == 0));
#pragma unroll
  for (int d = 0; d < NV; ++d)
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      const int c = d * 32 + 8 * w + 4 * g;
      if (c >= sh.vdim) continue;
      float o[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) o[e] = acc[d][4 * w + e] * inv;
      if (vec) {
        if (gate) {
          float z[4];
          ldv<4, T>(gate + c, z);
#pragma unroll
          for (int e = 0; e < 4; ++e) o[e] *= sigmoid_f(z[e]);
        }
        stv<4, T>(op + c, o);
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (c + e < sh.vdim)
            op[c + e] = from_f<T>(gate ? o[e] * sigmoid_f(to_f(gate[c + e])) : o[e]);
      }
    }
}

template <typename T, int NK, int NV>
int launch_prefill(const T* q, const T* kc, const T* vc, const T* proj, long ld, int g_col, T* out,
                   const SeqSpan* seqs, int n_seqs, int max_n, const AttnShape& sh,
                   const AttnMask& mask, hipStream_t s) {
  constexpr int V = FT<T>::kVec;
  constexpr size_t smem = sizeof(T) * ((size_t)kKT * (NK * 32 + V) +
                                       (size_t)NV * 32 * (kKT + 16 / sizeof(T)));
  auto kern = attn_prefill_kernel<T, NK, NV>;
  if (smem > 48 * 1024) {
    if (int rc = lsh_check_hip(hipFuncSetAttribute(reinterpret_cast<const void*>(kern),
                                                   hipFuncAttributeMaxDynamicSharedMemorySize,
                                                   (int)smem),
                               "hipFuncSetAttribute(attn_prefill)"))
      return rc;
  }
  const dim3 grid((max_n + kQT - 1) / kQT, sh.heads, n_seqs);
  kern<<<grid, 256, smem, s>>>(q, kc, vc, proj, ld, g_col, out, seqs, sh, mask);
  return lsh_check_launch("attn_prefill_kernel");
}

// ------------------------------------------------------------------------------------------------
// One-token kernel.  A workgroup of 8 wavefronts takes up to R query heads of one (row, kv head) and
// one part of the visible keys (numbered 0 .. n_vis - 1, the kept ones first).  16 lanes share a key;
// such a group keeps the running soft-max of the keys it has seen in registers, so nothing is
// exchanged until the end, and it requests the keys and values of its next turn before it computes
// on the present ones.
constexpr int kDecThreads = 512, kDecGroups = kDecThreads / 16;

// N consecutive elements in 4-byte words, converted when they are used
template <typename T, int N>
struct Packed {
  static constexpr int W = N * (int)sizeof(T) / 4;
  uint32_t w[W];
  __device__ __forceinline__ void load(const T* p) {  // 4-byte aligned
    if constexpr (W % 4 == 0) {
#pragma unroll
      for (int i = 0; i < W; i += 4) {
        const frag_t t = *reinterpret_cast<const frag_t*>(reinterpret_cast<const uint32_t*>(p) + i);
#pragma unroll
        for (int k = 0; k < 4; ++k) w[i + k] = t[k];
      }
    } else if constexpr (W % 2 == 0) {
#pragma unroll
      for (int i = 0; i < W; i += 2) {
        const uint2 t = *reinterpret_cast<const uint2*>(reinterpret_cast<const uint32_t*>(p) + i);
        w[i] = t.x;
        w[i + 1] = t.y;
      }
    } else {
#pragma unroll
      for (int i = 0; i < W; ++i) w[i] = reinterpret_cast<const uint32_t*>(p)[i];
    }
  }
  __device__ __forceinline__ void store(T* p) const {
#pragma unroll
    for (int i = 0; i < W; ++i) reinterpret_cast<uint32_t*>(p)[i] = w[i];
  }
  __device__ __forceinline__ float get(int e) const {
    if constexpr (sizeof(T) == 4) return __builtin_bit_cast(float, w[e]);
    else return __builtin_bit_cast(float, e & 1 ? w[e >> 1] & 0xffff0000u : w[e >> 1] << 16);
  }
};

// Where the queries lie, and (new_k; only where the values are the keys) the position's own key when
// the cache does not hold it yet: every workgroup takes it from there, one of them appends it.
template <typename T>
struct DecodeSource {
  const T* q;
  long q_ld, q_head;  // elements from row to row, from head to head
  const T* new_k;
  long k_ld;
};

// EK, EV: elements per lane of a key / value row; SAME: the values are the keys, read once
template <typename T, int EK, int EV, int R, bool SAME>
__global__ void __launch_bounds__(kDecThreads)
attn_decode_kernel(DecodeSource<T> src, const T* __restrict__ k_cache,
                   const T* __restrict__ v_cache, const T* __restrict__ proj, long ld, int g_col,
                   T* __restrict__ out, const int* __restrict__ row_slot,
                   const int* __restrict__ row_pos, int nsplit, int head_groups,
                   float* __restrict__ workspace, AttnShape sh, AttnMask mask) {
  constexpr int DP = EK * 16, VP = EV * 16;
  constexpr int U = (EK + EV) * (int)sizeof(T) > 64 ? 2 : 4;  // keys per group and turn
  __shared__ float part[8][R][VP], pm[8][R], pl[8][R];
  const int row = blockIdx.x, kvh = blockIdx.y / head_groups, hg = blockIdx.y % head_groups;
  const int split = blockIdx.z;
  const int rep = sh.heads / sh.kv_heads;
  const int h0 = kvh * rep + hg * R, nh = min(R, rep - hg * R);
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, grp = tid >> 4, j = tid & 15;
  const int pos = row_pos[row];
  const long cache0 = ((long)row_slot[row] * sh.kv_heads + kvh) * sh.max_step;
  const T* kc = k_cache + cache0 * DP + j * EK;
  const T* vc = v_cache + cache0 * VP + j * EV;
  const T* nk = SAME && src.new_k ? src.new_k + row * src.k_ld + kvh * DP + j * EK : nullptr;
  static_assert(!SAME || EK == EV, "values of the keys' size");
  const int lo = mask.first_seen(pos);  // first key of the window
  const int kept = min(mask.keep_first, lo);                           // kept keys before it
  const int n_vis = kept + pos + 1 - lo;
  const int per = ((n_vis + nsplit - 1) / nsplit + 15) & ~15;
  const int v_lo = min(split * per, n_vis), v_hi = min(v_lo + per, n_vis);

  Packed<T, EK> kb[2][U];
  Packed<T, EV> vb[2][U];
  auto fetch = [&](int c0, Packed<T, EK> (&ko)[U], Packed<T, EV> (&vo)[U]) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int v = min(c0 + u * kDecGroups + grp, v_hi - 1);
      const long key = v < kept ? v : lo + v - kept;
      if constexpr (SAME) ko[u].load(nk && key == pos ? nk : kc + key * DP);
      else ko[u].load(kc + key * DP);
      if constexpr (!SAME) vo[u].load(vc + key * VP);
    }
  };
  if (v_lo < v_hi) fetch(v_lo, kb[0], vb[0]);

  float qv[R][EK], acc[R][EV], m[R], l[R];
#pragma unroll
  for (int r = 0; r < R; ++r) {
    Packed<T, EK> t;
    t.load(src.q + row * src.q_ld + (h0 + min(r, nh - 1)) * src.q_head + j * EK);
#pragma unroll
    for (int e = 0; e < EK; ++e) qv[r][e] = t.get(e) * (mask.scale * kLog2e);
#pragma unroll
    for (int e = 0; e < EV; ++e) acc[r][e] = 0.f;
    m[r] = -INFINITY;
    l[r] = 0.f;
  }
  auto turn = [&](int c0, const Packed<T, EK> (&ki)[U], const Packed<T, EV> (&vi)[U]) {
    float s[U][R];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const bool in = c0 + u * kDecGroups + grp < v_hi;
#pragma unroll
      for (int r = 0; r < R; ++r) {
        float d = 0.f;
#pragma unroll
        for (int e = 0; e < EK; ++e) d = fmaf(qv[r][e], ki[u].get(e), d);
        d += dpp_f<kDppXor1>(d);
        d += dpp_f<kDppXor2>(d);
        d += dpp_f<kDppHalfMirror>(d);
        d += dpp_f<kDppMirror>(d);
        s[u][r] = in ? d : -INFINITY;
      }
    }
#pragma unroll
    for (int r = 0; r < R; ++r) {
      float mx = m[r];
#pragma unroll
      for (int u = 0; u < U; ++u) mx = fmaxf(mx, s[u][r]);
      const float ref = mx == -INFINITY ? 0.f : mx;  // nothing seen yet: all weights are zero
      const float f = exp2_f(m[r] - ref);
      m[r] = mx;
      l[r] *= f;
#pragma unroll
      for (int e = 0; e < EV; ++e) acc[r][e] *= f;
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const float p = exp2_f(s[u][r] - ref);
        l[r] += p;
#pragma unroll
        for (int e = 0; e < EV; ++e) acc[r][e] = fmaf(p, SAME ? ki[u].get(e) : vi[u].get(e), acc[r][e]);
      }
    }
  };
  constexpr int STEP = U * kDecGroups;
  for (int c0 = v_lo; c0 < v_hi; c0 += 2 * STEP) {
    if (c0 + STEP < v_hi) fetch(c0 + STEP, kb[1], vb[1]);
    turn(c0, kb[0], vb[0]);
    if (c0 + STEP < v_hi) {
      if (c0 + 2 * STEP < v_hi) fetch(c0 + 2 * STEP, kb[0], vb[0]);
      turn(c0 + STEP, kb[1], vb[1]);
    }
  }
  if constexpr (SAME) {
    if (nk && hg == 0 && split == 0 && grp == 0) {  // read from the cache by later launches only
      Packed<T, EK> t;
      t.load(nk);
      t.store(const_cast<T*>(kc) + (long)pos * DP);
    }
  }
  // merge the groups: the wavefront's four by lane exchange, the wavefronts over LDS
#pragma unroll
  for (int r = 0; r < R; ++r) {
    float mx = fmaxf(m[r], __shfl_xor(m[r], 16));
    mx = fmaxf(mx, __shfl_xor(mx, 32));
    const float f = m[r] == -INFINITY ? 0.f : exp2_f(m[r] - mx);
    float t = l[r] * f;
    t += __shfl_xor(t, 16);
    t += __shfl_xor(t, 32);
#pragma unroll
    for (int e = 0; e < EV; ++e) {
      float a = acc[r][e] * f;
      a += __shfl_xor(a, 16);
      a += __shfl_xor(a, 32);
      if (lane < 16) part[wave][r][j * EV + e] = a;
    }
    if (lane == 0) {
      pm[wave][r] = mx;
      pl[wave][r] = t;
    }
  }
  __syncthreads();
  const bool sink = mask.sink && split == 0;
  for (int x = tid; x < nh * VP; x += kDecThreads) {
    const int r = x / VP, c = x - r * VP;
    const float sink2 = sink && mask.sinks ? mask.sinks[h0 + r] * kLog2e : 0.f;
    float mx = sink ? sink2 : -INFINITY;
#pragma unroll
    for (int w = 0; w < 8; ++w) mx = fmaxf(mx, pm[w][r]);
    float a = 0.f, t = sink ? exp2_f(sink2 - mx) : 0.f;
#pragma unroll
    for (int w = 0; w < 8; ++w) {
      const float f = pm[w][r] == -INFINITY ? 0.f : exp2_f(pm[w][r] - mx);
      a = fmaf(f, part[w][r][c], a);
      t = fmaf(f, pl[w][r], t);
    }
    const int head = h0 + r;
    if (nsplit > 1) {
      // [row][head][split][VP + 2]: context, maximum, sum
      float* ws = workspace + (((long)row * sh.heads + head) * nsplit + split) * (VP + 2);
      ws[c] = a;
      if (c == 0) {
        ws[VP] = mx;
        ws[VP + 1] = t;
      }
    } else if (c < sh.vdim) {
      float o = a / t;
      if (g_col >= 0) o *= sigmoid_f(to_f(proj[(long)row * ld + g_col + head * sh.vdim + c]));
      out[(long)row * sh.heads * sh.vdim + head * sh.vdim + c] = from_f<T>(o);
    }
  }
}

template <typename T>
__global__ void __launch_bounds__(256)
attn_decode_combine_kernel(const float* __restrict__ workspace, const T* __restrict__ proj, long ld,
                           int g_col, T* __restrict__ out, int nsplit, int vp, AttnShape sh) {
  const int row = blockIdx.x, head = blockIdx.y;
  const float* w = workspace + ((long)row * sh.heads + head) * nsplit * (vp + 2);
  float m = -INFINITY;
  for (int p = 0; p < nsplit; ++p) m = fmaxf(m, w[(long)p * (vp + 2) + vp]);
  for (int c = threadIdx.x; c < sh.vdim; c += blockDim.x) {
    float a = 0.f, l = 0.f;
    for (int p = 0; p < nsplit; ++p) {
      const float* wp = w + (long)p * (vp + 2);
      const float f = wp[vp] == -INFINITY ? 0.f : exp2_f(wp[vp] - m);
      a += f * wp[c];
      l += f * wp[vp + 1];
    }
    float o = a / l;
    if (g_col >= 0) o *= sigmoid_f(to_f(proj[(long)row * ld + g_col + head * sh.vdim + c]));
    out[(long)row * sh.heads * sh.vdim + head * sh.vdim + c] = from_f<T>(o);
  }
}

constexpr int kMaxSplit = 32;

int check_shape(const AttnShape& sh, const char* who) {
  if (sh.heads <= 0 || sh.kv_heads <= 0 || sh.heads % sh.kv_heads != 0 || sh.max_step <= 0)
    return lsh_fail(LSH_ERR_INVALID, who);
  if (attn_pad(sh.dim) == 0 || attn_pad(sh.vdim) == 0 || sh.dim_pad != attn_pad(sh.dim) ||
      sh.vdim_pad != attn_pad(sh.vdim))
    return lsh_fail(LSH_ERR_UNSUPPORTED, "attention: head sizes above 256");
  return LSH_OK;
}

}  // namespace

template <typename T>
int attn_prepare(const T* proj, long ld, int q_col, int k_col, int v_col, const float* q_norm,
                 const float* k_norm, float eps, const float2* cos_sin, int rot_pairs, T* q_out,
                 T* k_cache, T* v_cache, const int* row_slot, const int* row_pos, int rows,
                 const AttnShape& sh, hipStream_t s) {
  if (int rc = check_shape(sh, "attn_prepare: bad shape")) return rc;
  const bool own = k_col >= 0, values = own && v_col >= 0;
  if (!proj || !q_out || !row_slot || !row_pos || rows <= 0 || rot_pairs < 0 ||
      2 * rot_pairs > sh.dim || (rot_pairs > 0 && !cos_sin) || (own && !k_cache) ||
      (values && !v_cache))
    return lsh_fail(LSH_ERR_INVALID, "attn_prepare: bad arguments");
  const int per_row = sh.heads + (own ? sh.kv_heads : 0) + (values ? sh.kv_heads : 0);
  const long units = (long)rows * per_row;
  if (sh.dim % 4 == 0 && ld % 4 == 0 && q_col % 4 == 0 && units < (1L << 24) &&
      (!own || k_col % 4 == 0) && (!values || (sh.vdim % 4 == 0 && v_col % 4 == 0))) {
    const int pad = values ? std::max(sh.dim_pad, sh.vdim_pad) : sh.dim_pad;
#define PREP4(LPH)                                                                              \
  attn_prepare4_kernel<T, LPH><<<(unsigned)((units * LPH + 255) / 256), 256, 0, s>>>(           \
      proj, ld, q_col, k_col, v_col, q_norm, k_norm, eps, cos_sin, rot_pairs, q_out, k_cache,   \
      v_cache, row_slot, row_pos, (int)units, per_row, sh)
    if (pad <= 64) PREP4(16);
    else if (pad <= 128) PREP4(32);
    else PREP4(64);
#undef PREP4
    return lsh_check_launch("attn_prepare4_kernel");
  }
  attn_prepare_kernel<T><<<(unsigned)((units + 3) / 4), 256, 0, s>>>(
      proj, ld, q_col, k_col, v_col, q_norm, k_norm, eps, cos_sin, rot_pairs, q_out, k_cache,
      v_cache, row_slot, row_pos, units, per_row, sh);
  return lsh_check_launch("attn_prepare_kernel");
}

#define PICK_V(NK)                                                                              \
  switch (sh.vdim_pad / 32) {                                                                   \
    case 2: return launch_prefill<T, NK, 2>(q, k_cache, v_cache, proj, ld, g_col, out, seqs,    \
                                            n_seqs, max_n, sh, mask, s);                        \
    case 3: return launch_prefill<T, NK, 3>(q, k_cache, v_cache, proj, ld, g_col, out, seqs,    \
                                            n_seqs, max_n, sh, mask, s);                        \
    case 4: return launch_prefill<T, NK, 4>(q, k_cache, v_cache, proj, ld, g_col, out, seqs,    \
                                            n_seqs, max_n, sh, mask, s);                        \
    default: return launch_prefill<T, NK, 8>(q, k_cache, v_cache, proj, ld, g_col, out, seqs,   \
                                             n_seqs, max_n, sh, mask, s);                       \
  }

template <typename T>
int attn_prefill(const T* q, const T* k_cache, const T* v_cache, const T* proj, long ld, int g_col,
                 T* out, const SeqSpan* seqs, int n_seqs, int max_n, const AttnShape& sh,
                 const AttnMask& mask, hipStream_t s) {
  if (int rc = check_shape(sh, "attn_prefill: bad shape")) return rc;
  if (!q || !k_cache || !v_cache || !out || !seqs || n_seqs <= 0 || max_n <= 0 ||
      (g_col >= 0 && !proj) || n_seqs > 65535 || sh.heads > 65535 ||
      (v_cache == k_cache && sh.dim != sh.vdim) || mask.chunk < 0)
    return lsh_fail(LSH_ERR_INVALID, "attn_prefill: bad arguments");
  switch (sh.dim_pad / 32) {
    case 2: PICK_V(2)
    case 3: PICK_V(3)
    case 4: PICK_V(4)
    default: PICK_V(8)
  }
}

size_t attn_decode_workspace(int rows, const AttnShape& sh) {
  return (size_t)rows * sh.heads * kMaxSplit * (sh.vdim_pad + 2);
}

#define DEC(EK, EV, R, SAME)                                                                     \
  attn_decode_kernel<T, EK, EV, R, SAME><<<grid, kDecThreads, 0, s>>>(                           \
      src, k_cache, v_cache, proj, ld, g_col, out, row_slot, row_pos, nsplit, groups, workspace,   \
      sh, mask)
#define DEC_R(EK, EV, SAME)                                                                      \
  do {                                                                                           \
    if (R == 1) DEC(EK, EV, 1, SAME);                                                            \
    else if (R == 2) DEC(EK, EV, 2, SAME);                                                       \
    else DEC(EK, EV, 4, SAME);                                                                   \
  } while (0)
#define DEC_V(EK)                                                                                \
  if (v_cache == k_cache) DEC_R(EK, EK, true);                                                   \
  else switch (sh.vdim_pad / 16) {                                                               \
    case 4: DEC_R(EK, 4, false); break;                                                          \
    case 6: DEC_R(EK, 6, false); break;                                                          \
    case 8: DEC_R(EK, 8, false); break;                                                          \
    default: DEC_R(EK, 16, false); break;                                                        \
  }

namespace {

template <typename T>
int launch_decode(const DecodeSource<T>& src, const T* k_cache, const T* v_cache, const T* proj, long ld,
                  int g_col, T* out, const int* row_slot, const int* row_pos, int rows, int max_len,
                  float* workspace, const AttnShape& sh, const AttnMask& mask, hipStream_t s) {
  if (int rc = check_shape(sh, "attn_decode: bad shape")) return rc;
  if (!src.q || !k_cache || !v_cache || !out || !row_slot || !row_pos || rows <= 0 || max_len <= 0 ||
      !workspace || (g_col >= 0 && !proj) || (v_cache == k_cache && sh.dim != sh.vdim) ||
      mask.chunk < 0)
    return lsh_fail(LSH_ERR_INVALID, "attn_decode: bad arguments");
  const int rep = sh.heads / sh.kv_heads;
  // heads per workgroup: several share the loads of a key, but only as many as leave the chip filled
  // (the kernel's time is the arithmetic of the compute units that work)
  const long each = (long)rows * sh.kv_heads, fill = 2L * cu_count();
  const int R = rep == 1 || each * rep <= fill ? 1 : rep == 2 || each * ((rep + 1) / 2) <= fill ? 2 : 4;
  const int groups = (rep + R - 1) / R;
  long most = max_len;
  if (mask.window > 0) most = std::min(most, (long)mask.window + mask.keep_first);
  if (mask.chunk > 0) most = std::min(most, (long)mask.chunk + mask.keep_first);
  // enough workgroups to fill the chip, but parts of at least 1024 keys: a shorter part is done
  // before the launch that would join the parts has started
  const int want = (int)((2L * cu_count() + (long)rows * sh.kv_heads * groups - 1) /
                         ((long)rows * sh.kv_heads * groups));
  const int nsplit = (int)std::max(1L, std::min({(long)kMaxSplit, (long)want, most / 1024}));
  if ((long)sh.kv_heads * groups > 65535) return lsh_fail(LSH_ERR_UNSUPPORTED, "attn_decode: heads");
  const dim3 grid(rows, sh.kv_heads * groups, nsplit);
  switch (sh.dim_pad / 16) {
    case 4: DEC_V(4) break;
    case 6: DEC_V(6) break;
    case 8: DEC_V(8) break;
    default: DEC_V(16) break;
  }
  if (int rc = lsh_check_launch("attn_decode_kernel")) return rc;
  if (nsplit > 1) {
    attn_decode_combine_kernel<T><<<dim3(rows, sh.heads), sh.vdim <= 64 ? 64 : 128, 0, s>>>(
        workspace, proj, ld, g_col, out, nsplit, sh.vdim_pad, sh);
    return lsh_check_launch("attn_decode_combine_kernel");
  }
  return LSH_OK;
}

}  // namespace

template <typename T>
int attn_decode(const T* q, const T* k_cache, const T* v_cache, const T* proj, long ld, int g_col,
                T* out, const int* row_slot, const int* row_pos, int rows, int max_len,
                float* workspace, const AttnShape& sh, const AttnMask& mask, hipStream_t s) {
  return launch_decode<T>(DecodeSource<T>{q, (long)sh.heads * sh.dim_pad, sh.dim_pad, nullptr, 0},
                          k_cache, v_cache, proj, ld, g_col, out, row_slot, row_pos, rows, max_len,
                          workspace, sh, mask, s);
}

bool attn_decode_append_supported(const AttnShape& sh, int q_col, int k_col, long ld) {
  return sh.dim == sh.vdim && sh.dim == sh.dim_pad && (q_col | k_col) % 8 == 0 && ld % 8 == 0;
}

template <typename T>
int attn_decode_append(const T* proj, long ld, int q_col, int k_col, T* k_cache, T* out,
                       const int* row_slot, const int* row_pos, int rows, int max_len,
                       float* workspace, const AttnShape& sh, const AttnMask& mask, hipStream_t s) {
  if (!proj || q_col < 0 || k_col < 0 || (reinterpret_cast<uintptr_t>(proj) & 15u) != 0)
    return lsh_fail(LSH_ERR_INVALID, "attn_decode_append: bad arguments");
  if (!attn_decode_append_supported(sh, q_col, k_col, ld))
    return lsh_fail(LSH_ERR_UNSUPPORTED, "attn_decode_append: head sizes or columns need padding");
  return launch_decode<T>(DecodeSource<T>{proj + q_col, ld, sh.dim, proj + k_col, ld}, k_cache,
                          k_cache, nullptr, 0, -1, out, row_slot, row_pos, rows, max_len, workspace,
                          sh, mask, s);
}

#define INST(T)                                                                                   \
  template int attn_prepare<T>(const T*, long, int, int, int, const float*, const float*, float,  \
                               const float2*, int, T*, T*, T*, const int*, const int*, int,       \
                               const AttnShape&, hipStream_t);                                    \
  template int attn_prefill<T>(const T*, const T*, const T*, const T*, long, int, T*,             \
                               const SeqSpan*, int, int, const AttnShape&, const AttnMask&,       \
                               hipStream_t);                                                      \
  template int attn_decode<T>(const T*, const T*, const T*, const T*, long, int, T*, const int*,  \
                              const int*, int, int, float*, const AttnShape&, const AttnMask&,    \
                              hipStream_t);                                                       \
  template int attn_decode_append<T>(const T*, long, int, int, T*, T*, const int*, const int*,    \
                                     int, int, float*, const AttnShape&, const AttnMask&,         \
                                     hipStream_t);
INST(float)
INST(bf16_t)

}  // namespace lsh
