// Gated linear attention:  S <- diag(a) S + k v^T;  o = S^T q  per head, with one decay per key channel,
// a = sigmoid(A2 low + bias)^(1 / tau).  State, decays and every product of the recurrence are
// float32; q, k, v and the output gate are read from the projection as they lie there.
//
//  * gla_scan_kernel   -- token by token, any size: decays, recurrence, read-out, head norm and output
//    gate in one launch, the state in registers.  One token per sequence is its shortest case.
//  * gla_chunk_*       -- a prompt in chunks of 64 tokens, sub-blocks of 16.  With b the running sum of
//    log a inside a chunk and S the state before it,
//      o_t = S^T (q_t e^(b_t)) + sum_{j <= t} [sum_d q_td k_jd e^(b_td - b_jd)] v_j,
//      S  <- e^(b_64) S + sum_j (k_j e^(b_64 - b_j)) v_j^T.
//    What a chunk adds to the state does not depend on the state, so one launch forms it for all
//    chunks at once, a second adds the chunks up (element by element) and leaves the state before each,
//    a third computes the outputs of all chunks at once.  Between sub-blocks the exponent is split at
//    the end of the keys' block, inside one the decays are multiplied up token by token: no exponent
//    is ever positive.
//
// Lane layout of the chunk kernels: wavefront w has the tokens 16 w .. 16 w + 15 of its chunk; lane
// (c = lane % 16, qd = lane / 16) holds token c's channels 16 s + 4 qd .. + 3 for every s.  That is an
// operand of the float32 matrix product and, for the decays, the result of one; moving along the
// tokens is a shift within 16 lanes.
#include <algorithm>

#include "lm_launch.h"

namespace lsh {

namespace {

constexpr int kC = 64;

__device__ __forceinline__ float exp2_f(float x) { return __builtin_amdgcn_exp2f(x); }
// log2 of sigmoid(z)^(1 / tau) = -(max(-z, 0) log2(e) + log2(1 + u)) / tau with u = e^-|z|.  The sum 1 + u
// loses the low bits of a small u; scaling its logarithm by u / ((1 + u) - 1) puts them back.
__device__ __forceinline__ float log2_decay(float z, float inv_tau) {
  constexpr float kLog2e = 1.44269504088896340736f;
  const float u = exp2_f(-fabsf(z) * kLog2e), w = 1.f + u, d = w - 1.f;
  const float l = d == 0.f ? u * kLog2e : __builtin_amdgcn_logf(w) * (u * __builtin_amdgcn_rcpf(d));
  return -(fmaxf(-z, 0.f) * kLog2e + l) * inv_tau;
}

// a lane's value from N lanes before (after) it in its row of 16, zero at the border (a form that the
// compiler folds into the operation that uses it)
template <int CTRL>
__device__ __forceinline__ float row_shift(float x) {
  return __builtin_bit_cast(
      float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, x), CTRL, 0xf, 0xf, true));
}
template <int N>
__device__ __forceinline__ float lanes_before(float x) {
  if constexpr (N == 0) return x;
  else return row_shift<0x110 + N>(x);
}
template <int N>
__device__ __forceinline__ float lanes_after(float x) {
  return row_shift<0x100 + N>(x);
}

template <typename T>
__device__ __forceinline__ f32x4 load4(const T* p) {
  float t[4];
  ldv<4, T>(p, t);
  return f32x4{t[0], t[1], t[2], t[3]};
}
__device__ __forceinline__ frag_t as_frag(f32x4 x) { return __builtin_bit_cast(frag_t, x); }
__device__ __forceinline__ frag_t ldfrag(const float* p) { return *reinterpret_cast<const frag_t*>(p); }
__device__ __forceinline__ f32x4 exp4(f32x4 x) {  // 2^x
  return f32x4{exp2_f(x[0]), exp2_f(x[1]), exp2_f(x[2]), exp2_f(x[3])};
}

// ------------------------------------------------------------------------------------------------
// One workgroup per (sequence, head).  LPD lanes share a row of the state (one value channel, V == 4:
// four adjacent key channels per lane, else every LPD-th), a thread has at most RM rows.
template <typename T, int V, int LPD, int RM, int NTH>
__global__ void __launch_bounds__(NTH)
gla_scan_kernel(const T* __restrict__ proj, long ld, const float* __restrict__ low, GlaWeights wt,
                float* __restrict__ state, T* __restrict__ out, const SeqSpan* __restrict__ seqs,
                const int* __restrict__ row_slot, const int* __restrict__ row_pos, GlaShape sh) {
  constexpr int NVG = NTH / LPD;
  __shared__ float as[256], qs[256], ks[256], vs[256], os[256], red[16];
  const int D = sh.dim, VD = sh.vdim, H = sh.heads, h = blockIdx.y;
  const int tid = threadIdx.x, l = tid % LPD, vg = tid / LPD;
  SeqSpan sq;
  if (seqs) sq = seqs[blockIdx.x];
  else sq = SeqSpan{(int)blockIdx.x, 1, row_pos[blockIdx.x], row_slot[blockIdx.x]};
  const auto channel = [&](int e) { return V == 4 ? 4 * l + e : l + LPD * e; };
  float* sp = state + ((long)sq.slot * H + h) * VD * D;
  float S[RM][4];
#pragma unroll
  for (int i = 0; i < RM; ++i) {
    const int v = vg + NVG * i;
#pragma unroll
    for (int e = 0; e < 4; ++e) S[i][e] = 0.f;
    if (sq.pos0 > 0 && v < VD) {
      if (V == 4) {
        if (4 * l < D) ldv<4, float>(sp + (long)v * D + 4 * l, S[i]);
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (channel(e) < D) S[i][e] = sp[(long)v * D + channel(e)];
      }
    }
  }
  const float qscale = 1.0f / sqrtf((float)D);
  for (int t = 0; t < sq.n; ++t) {
    const long row = sq.row0 + t;
    const T* pr = proj + row * ld;
    const float gate = tid < VD ? to_f(pr[sh.g_col + h * VD + tid]) : 0.f;
    for (int x = tid; x < 3 * D + VD; x += NTH) {
      if (x < D) {
        const float *a2 = wt.a2 + (long)(h * D + x) * sh.rank, *lr = low + row * sh.rank;
        float z = wt.bias[h * D + x];
        for (int r = 0; r < sh.rank; r += 4) {
          const f32x4 a = load4(a2 + r), b = load4(lr + r);
#pragma unroll
          for (int e = 0; e < 4; ++e) z = fmaf(a[e], b[e], z);
        }
        as[x] = exp2_f(log2_decay(z, sh.inv_tau));
      } else if (x < 2 * D) {
        qs[x - D] = to_f(pr[sh.q_col + h * D + x - D]) * qscale;
      } else if (x < 3 * D) {
        ks[x - 2 * D] = to_f(pr[sh.k_col + h * D + x - 2 * D]);
      } else {
        vs[x - 3 * D] = to_f(pr[sh.v_col + h * VD + x - 3 * D]);
      }
    }
    __syncthreads();
    float a[4], q[4], k[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int d = channel(e);
      const bool in = d < D;
      a[e] = in ? as[d] : 0.f;
      q[e] = in ? qs[d] : 0.f;
      k[e] = in ? ks[d] : 0.f;
    }
#pragma unroll
    for (int i = 0; i < RM; ++i) {
      const int v = vg + NVG * i;
      const float vv = v < VD ? vs[v] : 0.f;
      float o = 0.f;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        S[i][e] = fmaf(k[e], vv, a[e] * S[i][e]);
        o = fmaf(q[e], S[i][e], o);
      }
      o += dpp_f<kDppXor1>(o);
      o += dpp_f<kDppXor2>(o);
      o += dpp_f<kDppHalfMirror>(o);
      o += dpp_f<kDppMirror>(o);
      if (LPD > 16) o += __shfl_xor(o, 16);
      if (LPD > 32) o += __shfl_xor(o, 32);
      if (l == 0 && v < VD) os[v] = o;
    }
    __syncthreads();
    const float o = tid < VD ? os[tid] : 0.f;
    const float ss = block_sum_dpp(o * o, red);
    if (tid < VD) {
      const float r = 1.0f / sqrtf(ss / (float)VD + sh.eps);
      out[(row * H + h) * VD + tid] = from_f<T>(o * r * wt.norm[tid] * silu_f(gate));
    }
  }
#pragma unroll
  for (int i = 0; i < RM; ++i) {
    const int v = vg + NVG * i;
    if (v >= VD) continue;
    if (V == 4) {
      if (4 * l < D) stv<4, float>(sp + (long)v * D + 4 * l, S[i]);
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (channel(e) < D) sp[(long)v * D + channel(e)] = S[i][e];
    }
  }
}

// ------------------------------------------------------------------------------------------------
// Workspace of one (chunk, head): what the chunk adds to the state, then the state before it; the
// chunk's decay [D].  Chunk c of a sequence is number row0 / 64 + sequence index + c.  The state is cut
// into blocks of 16 x 16 (value block vb, slice s: number vb * (D / 16) + s), each as the lanes of a
// wavefront hold it as an operand: lane (c, qd) value channel 16 vb + c, key channels 16 s + 4 qd .. + 3.
__host__ __device__ inline long chunk_floats(const GlaShape& sh) {
  return (long)sh.vdim * sh.dim + sh.dim;
}

// log2 decays of this lane's token and channels from slice s0 on; 0 for a token that is not there
template <int NS>
__device__ __forceinline__ void chunk_log_decays(const float* __restrict__ low, long row, bool in,
                                                 const GlaWeights& wt, const GlaShape& sh, int h, int s0,
                                                 int c, int qd, f32x4 (&la)[NS]) {
  const int ns = sh.dim / 16 - s0;
#pragma unroll
  for (int s = 0; s < NS; ++s) la[s] = (f32x4)0.f;
  for (int r = 0; r < sh.rank; r += 16) {
    const frag_t fl = ldfrag(low + row * sh.rank + r + qd * 4);
#pragma unroll
    for (int s = 0; s < NS; ++s)
      if (s < ns)
        la[s] = mma16(0.f, ldfrag(wt.a2 + (long)(h * sh.dim + (s0 + s) * 16 + c) * sh.rank + r + qd * 4), fl,
                      la[s]);
  }
#pragma unroll
  for (int s = 0; s < NS; ++s)
    if (s < ns) {
      const f32x4 b = load4(wt.bias + h * sh.dim + (s0 + s) * 16 + qd * 4);
#pragma unroll
      for (int e = 0; e < 4; ++e) la[s][e] = in ? log2_decay(la[s][e] + b[e], sh.inv_tau) : 0.f;
    }
}
// sums over the tokens of the sub-block up to this one / after this one
__device__ __forceinline__ f32x4 sum_upto(f32x4 x) {
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    x[e] += lanes_before<1>(x[e]);
    x[e] += lanes_before<2>(x[e]);
    x[e] += lanes_before<4>(x[e]);
    x[e] += lanes_before<8>(x[e]);
  }
  return x;
}
__device__ __forceinline__ f32x4 sum_after(f32x4 x) {
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    x[e] = lanes_after<1>(x[e]);
    x[e] += lanes_after<1>(x[e]);
    x[e] += lanes_after<2>(x[e]);
    x[e] += lanes_after<4>(x[e]);
    x[e] += lanes_after<8>(x[e]);
  }
  return x;
}

constexpr int kTS = kC + 4;  // row length of a matrix with the chunk's tokens as columns

// Values of a wavefront's blocks w, w + 4, .. as an operand: value channel c of its block, the tokens
// 16 J + 4 qd .. + 3.  A token that is not there is the last one again (its weights are zero).
template <typename T, int NVB>
struct ChunkValues {
  T x[NVB][4][4];
  __device__ __forceinline__ void fetch(const T* __restrict__ proj, long ld, long row0, int n,
                                        const GlaShape& sh, int h, int w, int c, int qd) {
#pragma unroll
    for (int b = 0; b < NVB; ++b)
      if ((w + 4 * b) * 16 < sh.vdim) {
        const T* src = proj + row0 * ld + sh.v_col + h * sh.vdim + (w + 4 * b) * 16 + c;
#pragma unroll
        for (int J = 0; J < 4; ++J)
#pragma unroll
          for (int j = 0; j < 4; ++j) x[b][J][j] = src[min(J * 16 + qd * 4 + j, n - 1) * ld];
      }
  }
  __device__ __forceinline__ frag_t frag(int b, int J) const {
    return as_frag(f32x4{to_f(x[b][J][0]), to_f(x[b][J][1]), to_f(x[b][J][2]), to_f(x[b][J][3])});
  }
};

// what a chunk adds to the state, and its decay
template <typename T, int NS>  // dim, vdim <= 16 * NS
__global__ void __launch_bounds__(256, NS <= 4 ? 4 : NS <= 8 ? 3 : 1)
gla_chunk_add_kernel(const T* __restrict__ proj, long ld, const float* __restrict__ low, GlaWeights wt,
                     float* __restrict__ ws, const SeqSpan* __restrict__ seqs, GlaShape sh) {
  constexpr int NVB = (NS + 3) / 4;  // value blocks of a wavefront
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const SeqSpan sq = seqs[blockIdx.z];
  const int c0 = blockIdx.x * kC;
  if (c0 >= sq.n) return;
  const int n = min(kC, sq.n - c0), h = blockIdx.y, H = sh.heads, D = sh.dim, VD = sh.vdim;
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, c = lane & 15, qd = lane >> 4;
  const int ns = D / 16, nv = VD / 16;
  float* Kt = sm;                 // [D][kTS]
  float* tot = Kt + D * kTS;      // [4][D]: log decay of every sub-block
  const long row0 = sq.row0 + c0;
  const int t = w * 16 + c;
  const bool in = t < n;
  const long row = row0 + min(t, n - 1);
  f32x4 k[NS], la[NS];
#pragma unroll
  for (int s = 0; s < NS; ++s)
    k[s] = s < ns && in ? load4(proj + row * ld + sh.k_col + h * D + s * 16 + qd * 4) : (f32x4)0.f;
  ChunkValues<T, NVB> values;
  values.fetch(proj, ld, row0, n, sh, h, w, c, qd);
  chunk_log_decays<NS>(low, row, in, wt, sh, h, 0, c, qd, la);
#pragma unroll
  for (int s = 0; s < NS; ++s)
    if (s < ns) {
      const f32x4 after = sum_after(la[s]);
      if (c == 0) *reinterpret_cast<f32x4*>(&tot[w * D + s * 16 + qd * 4]) = after + la[s];
      la[s] = after;
    }
  __syncthreads();
#pragma unroll
  for (int s = 0; s < NS; ++s)
    if (s < ns) {
      f32x4 left = la[s];
      for (int m = w + 1; m < 4; ++m) left += *reinterpret_cast<const f32x4*>(&tot[m * D + s * 16 + qd * 4]);
      const f32x4 x = k[s] * exp4(left);
#pragma unroll
      for (int e = 0; e < 4; ++e) Kt[(s * 16 + qd * 4 + e) * kTS + t] = x[e];
    }
  float* o = ws + ((sq.row0 / kC + (long)blockIdx.z + blockIdx.x) * H + h) * chunk_floats(sh);
  for (int d = tid; d < D; d += 256)
    o[(long)VD * D + d] = exp2_f((tot[d] + tot[D + d]) + (tot[2 * D + d] + tot[3 * D + d]));
  __syncthreads();
  for (int db = 0; db < ns; ++db) {
    frag_t fk[4];
#pragma unroll
    for (int J = 0; J < 4; ++J) fk[J] = ldfrag(&Kt[(db * 16 + c) * kTS + J * 16 + qd * 4]);
#pragma unroll
    for (int b = 0; b < NVB; ++b) {
      const int vb = w + 4 * b;
      if (vb >= nv) continue;
      f32x4 acc = (f32x4)0.f;
#pragma unroll
      for (int J = 0; J < 4; ++J) acc = mma16(0.f, fk[J], values.frag(b, J), acc);
      *reinterpret_cast<f32x4*>(&o[(vb * ns + db) * 256 + lane * 4]) = acc;
    }
  }
}

// adds the chunks of a sequence up; every chunk's place receives the state before it
__global__ void __launch_bounds__(256)
gla_chunk_state_kernel(float* __restrict__ ws, float* __restrict__ state,
                       const SeqSpan* __restrict__ seqs, GlaShape sh) {
  constexpr int U = 8;  // chunks requested at once
  const SeqSpan sq = seqs[blockIdx.z];
  const int h = blockIdx.y, H = sh.heads, D = sh.dim;
  const int x = (blockIdx.x * 256 + threadIdx.x) * 4, size = sh.vdim * D;
  if (x >= size) return;
  const long stride = H * chunk_floats(sh);
  float* base = ws + ((sq.row0 / kC + (long)blockIdx.z) * H + h) * chunk_floats(sh);
  const int lane = x / 4 % 64, block = x / 256, ns = D / 16;
  const int v = block / ns * 16 + lane % 16, d = block % ns * 16 + lane / 16 * 4;
  float* sp = state + ((long)sq.slot * H + h) * size + (long)v * D + d;
  const int chunks = (sq.n + kC - 1) / kC;
  f32x4 S = (f32x4)0.f;
  if (sq.pos0 > 0) S = load4(sp);
  for (int ch = 0; ch < chunks; ch += U) {
    f32x4 add[U], dec[U];
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (ch + u < chunks) {
        add[u] = load4(base + (ch + u) * stride + x);
        dec[u] = load4(base + (ch + u) * stride + size + d);
      }
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (ch + u < chunks) {
        *reinterpret_cast<f32x4*>(base + (ch + u) * stride + x) = S;
        S = dec[u] * S + add[u];
      }
  }
  *reinterpret_cast<f32x4*>(sp) = S;
}

// products inside a sub-block, x[DELTA] of p[t][t - DELTA] for rising DELTA; w carries q_t times the
// decays of the DELTA tokens up to t
template <int N, int DELTA>
__device__ __forceinline__ void diagonal(const f32x4 (&k)[N], const f32x4 (&a)[N], f32x4 (&w)[N],
                                         float (&x)[16]) {
  if constexpr (DELTA < 16) {
#pragma unroll
    for (int s = 0; s < N; ++s)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        x[DELTA] = fmaf(w[s][e], lanes_before<DELTA>(k[s][e]), x[DELTA]);
        if (DELTA < 15) w[s][e] *= lanes_before<DELTA>(a[s][e]);
      }
    diagonal<N, DELTA + 1>(k, a, w, x);
  }
}

// Outputs of a chunk, normed and gated.  First every wavefront forms the weights of its 16 tokens, then
// it takes value blocks w, w + 4, .. of all 64, so that state and values are read once.
template <typename T, int NS>  // dim, vdim <= 16 * NS
__global__ void __launch_bounds__(256, NS <= 4 ? 3 : NS <= 8 ? 2 : 1)
gla_chunk_out_kernel(const T* __restrict__ proj, long ld, const float* __restrict__ low, GlaWeights wt,
                     const float* __restrict__ ws, T* __restrict__ out,
                     const SeqSpan* __restrict__ seqs, GlaShape sh) {
  constexpr int GS = NS < 4 ? NS : 4;  // slices whose keys and decays are in registers at a time
  constexpr int NVB = (NS + 3) / 4;    // value blocks of a wavefront
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const SeqSpan sq = seqs[blockIdx.z];
  const int c0 = blockIdx.x * kC;
  if (c0 >= sq.n) return;
  const int n = min(kC, sq.n - c0), h = blockIdx.y, H = sh.heads, D = sh.dim, VD = sh.vdim;
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, c = lane & 15, qd = lane >> 4;
  const int ns = D / 16, nv = VD / 16, KS = D + 4;
  float* Q = sm;                 // [64][KS]: queries with their decays back to a block's end
  float* Kh = Q + kC * KS;       // [48][KS]: keys decayed to the end of their sub-block
  float* P = Kh + 48 * KS;       // [64][kTS]: weights of the chunk's tokens (lower blocks)
  float* Et = P + kC * kTS;      // [4][D]: decay of every sub-block
  float* sq_sum = Et + 4 * D;    // [4][64]
  const long row0 = sq.row0 + c0;
  const int t = w * 16 + c;
  const bool in = t < n;
  const long row = row0 + min(t, n - 1);
  const T* pr = proj + row * ld;
  const bool has_state = c0 > 0 || sq.pos0 > 0;
  {
    const float qscale = 1.0f / sqrtf((float)D);
    float x[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) x[i] = 0.f;
    // the next group's keys, queries and decays are under way while the present one is worked on
    typedef T T4 __attribute__((ext_vector_type(4)));
    T4 kn[GS], qn[GS];
    f32x4 ln[GS];
    const auto fetch = [&](int s0) {
#pragma unroll
      for (int s = 0; s < GS; ++s) {
        const int d = h * D + (s0 + s) * 16 + qd * 4;
        const bool there = s0 + s < ns && in;
        kn[s] = there ? *reinterpret_cast<const T4*>(pr + sh.k_col + d) : (T4)0.f;
        qn[s] = there ? *reinterpret_cast<const T4*>(pr + sh.q_col + d) : (T4)0.f;
      }
      chunk_log_decays<GS>(low, row, in, wt, sh, h, s0, c, qd, ln);
    };
    fetch(0);
#pragma unroll 1
    for (int s0 = 0; s0 < ns; s0 += GS) {
      f32x4 k[GS], la[GS], wq[GS];
#pragma unroll
      for (int s = 0; s < GS; ++s) {
        la[s] = ln[s];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          k[s][e] = to_f((T)kn[s][e]);
          wq[s][e] = to_f((T)qn[s][e]) * qscale;
        }
      }
      if (s0 + GS < ns) fetch(s0 + GS);
#pragma unroll
      for (int s = 0; s < GS; ++s)
        if (s0 + s < ns) {
          const int d = (s0 + s) * 16 + qd * 4;
          const f32x4 upto = exp4(sum_upto(la[s]));
          if (c == 15) *reinterpret_cast<f32x4*>(&Et[w * D + d]) = upto;
          if (w < 3) *reinterpret_cast<f32x4*>(&Kh[t * KS + d]) = k[s] * exp4(sum_after(la[s]));
          *reinterpret_cast<f32x4*>(&Q[t * KS + d]) = wq[s] * upto;
          la[s] = exp4(la[s]);
        }
      diagonal<GS, 0>(k, la, wq, x);
    }
    f32x4 p = (f32x4)0.f;
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      x[i] += __shfl_xor(x[i], 16);
      x[i] += __shfl_xor(x[i], 32);
#pragma unroll
      for (int e = 0; e < 4; ++e) p[e] = c - i == 4 * qd + e ? x[i] : p[e];
    }
    *reinterpret_cast<f32x4*>(&P[t * kTS + w * 16 + qd * 4]) = p;
  }
  __syncthreads();
  // earlier sub-blocks; q (this wavefront's rows only) is decayed further back with every one passed
  for (int J = w - 1; J >= 0; --J) {
    f32x4 pj = (f32x4)0.f;
#pragma unroll 4
    for (int s = 0; s < ns; ++s) {
      const int d = s * 16 + qd * 4;
      f32x4* qp = reinterpret_cast<f32x4*>(&Q[t * KS + d]);
      const f32x4 q = *qp;
      pj = mma16(0.f, ldfrag(&Kh[(J * 16 + c) * KS + d]), as_frag(q), pj);
      *qp = q * *reinterpret_cast<const f32x4*>(&Et[J * D + d]);
    }
    *reinterpret_cast<f32x4*>(&P[t * kTS + J * 16 + qd * 4]) = pj;
  }
  ChunkValues<T, NVB> values;
  values.fetch(proj, ld, row0, n, sh, h, w, c, qd);
  const float* S = ws + ((sq.row0 / kC + (long)blockIdx.z + blockIdx.x) * H + h) * chunk_floats(sh);
  __syncthreads();
  // transposed outputs: acc[b][I] has the value channels 16 (w + 4 b) + 4 qd .. + 3 of token 16 I + c
  f32x4 acc[NVB][4];
  float ss[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int b = 0; b < NVB; ++b) {
#pragma unroll
    for (int I = 0; I < 4; ++I) acc[b][I] = (f32x4)0.f;
    const int vb = w + 4 * b;
    if (vb >= nv) continue;
    if (has_state) {
      frag_t fs[NS];
#pragma unroll
      for (int s = 0; s < NS; ++s)
        if (s < ns) fs[s] = ldfrag(S + (vb * ns + s) * 256 + lane * 4);
#pragma unroll
      for (int s = 0; s < NS; ++s)
        if (s < ns) {
#pragma unroll
          for (int I = 0; I < 4; ++I)
            acc[b][I] = mma16(0.f, fs[s], ldfrag(&Q[(I * 16 + c) * KS + s * 16 + qd * 4]), acc[b][I]);
        }
    }
#pragma unroll
    for (int J = 0; J < 4; ++J) {
      const frag_t fv = values.frag(b, J);
#pragma unroll
      for (int I = J; I < 4; ++I)
        acc[b][I] = mma16(0.f, fv, ldfrag(&P[(I * 16 + c) * kTS + J * 16 + qd * 4]), acc[b][I]);
    }
#pragma unroll
    for (int I = 0; I < 4; ++I)
#pragma unroll
      for (int e = 0; e < 4; ++e) ss[I] += acc[b][I][e] * acc[b][I][e];
  }
#pragma unroll
  for (int I = 0; I < 4; ++I) {
    ss[I] += __shfl_xor(ss[I], 16);
    ss[I] += __shfl_xor(ss[I], 32);
    if (qd == 0) sq_sum[w * kC + I * 16 + c] = ss[I];
  }
  __syncthreads();
#pragma unroll
  for (int I = 0; I < 4; ++I) {
    const int ti = I * 16 + c;
    if (ti >= n) continue;
    const float sum = (sq_sum[ti] + sq_sum[kC + ti]) + (sq_sum[2 * kC + ti] + sq_sum[3 * kC + ti]);
    const float r = 1.0f / sqrtf(sum / (float)VD + sh.eps);
#pragma unroll
    for (int b = 0; b < NVB; ++b)
      if (w + 4 * b < nv) {
        const int vc = (w + 4 * b) * 16 + qd * 4;
        const f32x4 g = load4(proj + (row0 + ti) * ld + sh.g_col + h * VD + vc), nw = load4(wt.norm + vc);
        float o[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) o[e] = acc[b][I][e] * r * nw[e] * silu_f(g[e]);
        stv<4, T>(out + ((row0 + ti) * H + h) * VD + vc, o);
      }
  }
}

int check_shape(const GlaShape& sh) {
  if (sh.heads <= 0 || sh.heads > 65535 || sh.dim <= 0 || sh.vdim <= 0 || sh.rank <= 0 ||
      sh.rank % 16 != 0 || sh.q_col < 0 || sh.k_col < 0 || sh.v_col < 0 || sh.g_col < 0)
    return lsh_fail(LSH_ERR_INVALID, "gated linear attention: bad shape");
  if (sh.dim > 256 || sh.vdim > 256)
    return lsh_fail(LSH_ERR_UNSUPPORTED, "gated linear attention: head sizes above 256");
  return LSH_OK;
}

template <typename T>
int launch_scan(const T* proj, long ld, const float* low, const GlaWeights& w, float* state, T* out,
                const SeqSpan* seqs, const int* row_slot, const int* row_pos, int n,
                const GlaShape& sh, hipStream_t s) {
  const dim3 grid(n, sh.heads);
#define SCAN(V, LPD, RM, NTH)                                                                        \
  gla_scan_kernel<T, V, LPD, RM, NTH><<<grid, NTH, 0, s>>>(proj, ld, low, w, state, out, seqs,       \
                                                           row_slot, row_pos, sh)
#define SCAN_V(V)                                       \
  do {                                                  \
    if (sh.dim <= 64) {                                 \
      if (sh.vdim <= 64) SCAN(V, 16, 4, 256);           \
      else SCAN(V, 16, 16, 256);                        \
    } else if (sh.dim <= 128) {                         \
      if (sh.vdim <= 128) SCAN(V, 32, 16, 256);         \
      else SCAN(V, 32, 8, 1024);                        \
    } else {                                            \
      SCAN(V, 64, 16, 1024);                            \
    }                                                   \
  } while (0)
  if (sh.dim % 4 == 0) SCAN_V(4);
  else SCAN_V(1);
#undef SCAN_V
#undef SCAN
  return lsh_check_launch("gla_scan_kernel");
}

}  // namespace

template <typename T>
int gla_step(const T* proj, long ld, const float* low, const GlaWeights& w, float* state, T* out,
             const int* row_slot, const int* row_pos, int rows, const GlaShape& sh, hipStream_t s) {
  if (int rc = check_shape(sh)) return rc;
  if (!proj || !low || !w.a2 || !w.bias || !w.norm || !state || !out || !row_slot || !row_pos ||
      rows <= 0)
    return lsh_fail(LSH_ERR_INVALID, "gla_step: bad arguments");
  return launch_scan<T>(proj, ld, low, w, state, out, nullptr, row_slot, row_pos, rows, sh, s);
}

template <typename T>
int gla_scan(const T* proj, long ld, const float* low, const GlaWeights& w, float* state, T* out,
             const SeqSpan* seqs, int n_seqs, const GlaShape& sh, hipStream_t s) {
  if (int rc = check_shape(sh)) return rc;
  if (!proj || !low || !w.a2 || !w.bias || !w.norm || !state || !out || !seqs || n_seqs <= 0)
    return lsh_fail(LSH_ERR_INVALID, "gla_scan: bad arguments");
  return launch_scan<T>(proj, ld, low, w, state, out, seqs, nullptr, nullptr, n_seqs, sh, s);
}

// columns and rows of the projection in fours, head sizes in sixteens
bool gla_chunked_supported(const GlaShape& sh, long ld) {
  return sh.dim % 16 == 0 && sh.vdim % 16 == 0 && sh.dim <= 256 && sh.vdim <= 256 && ld % 4 == 0 &&
         (sh.q_col | sh.k_col | sh.v_col | sh.g_col) % 4 == 0;
}

size_t gla_chunked_workspace(int rows, int n_seqs, const GlaShape& sh) {
  return ((size_t)rows / kC + n_seqs) * sh.heads * chunk_floats(sh);
}

template <typename T>
int gla_chunked(const T* proj, long ld, const float* low, const GlaWeights& w, float* state, T* out,
                float* workspace, const SeqSpan* seqs, int n_seqs, int max_n, int rows,
                const GlaShape& sh, hipStream_t s) {
  if (int rc = check_shape(sh)) return rc;
  if (!proj || !low || !w.a2 || !w.bias || !w.norm || !state || !out || !workspace || !seqs ||
      n_seqs <= 0 || n_seqs > 65535 || max_n <= 0 || max_n > rows)
    return lsh_fail(LSH_ERR_INVALID, "gla_chunked: bad arguments");
  if (!gla_chunked_supported(sh, ld))
    return lsh_fail(LSH_ERR_UNSUPPORTED, "gla_chunked: head sizes must be multiples of 16");
  const dim3 grid((max_n + kC - 1) / kC, sh.heads, n_seqs);
  const int D = sh.dim, VD = sh.vdim, wide = std::max(D, VD);
  const auto room = [](const void* kernel, size_t lds) {
    return lsh_check_hip(hipFuncSetAttribute(kernel, hipFuncAttributeMaxDynamicSharedMemorySize,
                                             (int)lds),
                         "hipFuncSetAttribute(gla_chunk)");
  };
  {
    auto kern = wide <= 32 ? gla_chunk_add_kernel<T, 2> : wide <= 64 ? gla_chunk_add_kernel<T, 4>
              : wide <= 128 ? gla_chunk_add_kernel<T, 8> : gla_chunk_add_kernel<T, 16>;
    const size_t lds = sizeof(float) * ((size_t)D * kTS + 4 * D);
    if (int rc = room(reinterpret_cast<const void*>(kern), lds)) return rc;
    kern<<<grid, 256, lds, s>>>(proj, ld, low, w, workspace, seqs, sh);
    if (int rc = lsh_check_launch("gla_chunk_add_kernel")) return rc;
  }
  gla_chunk_state_kernel<<<dim3((VD * D / 4 + 255) / 256, sh.heads, n_seqs), 256, 0, s>>>(
      workspace, state, seqs, sh);
  if (int rc = lsh_check_launch("gla_chunk_state_kernel")) return rc;
  auto kern = wide <= 32 ? gla_chunk_out_kernel<T, 2> : wide <= 64 ? gla_chunk_out_kernel<T, 4>
            : wide <= 128 ? gla_chunk_out_kernel<T, 8> : gla_chunk_out_kernel<T, 16>;
  const size_t lds = sizeof(float) * ((size_t)(kC + 48) * (D + 4) + kC * kTS + 4 * D + 4 * kC);
  if (int rc = room(reinterpret_cast<const void*>(kern), lds)) return rc;
  kern<<<grid, 256, lds, s>>>(proj, ld, low, w, workspace, out, seqs, sh);
  return lsh_check_launch("gla_chunk_out_kernel");
}

#define INST(T)                                                                                     \
  template int gla_step<T>(const T*, long, const float*, const GlaWeights&, float*, T*, const int*, \
                           const int*, int, const GlaShape&, hipStream_t);                          \
  template int gla_scan<T>(const T*, long, const float*, const GlaWeights&, float*, T*,             \
                           const SeqSpan*, int, const GlaShape&, hipStream_t);                      \
  template int gla_chunked<T>(const T*, long, const float*, const GlaWeights&, float*, T*, float*,  \
                              const SeqSpan*, int, int, int, const GlaShape&, hipStream_t);
INST(float)
INST(bf16_t)

}  // namespace lsh
