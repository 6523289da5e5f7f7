// The gated delta rule:  S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q  per head, with
// unit q and k, after a short causal convolution of q, k and v.  State and everything that enters
// the recurrence are float32.
//
//  * delta_step_kernel   -- one token per sequence: convolution, gates, recurrence, read-out, head
//    norm and output gate in one launch; the state is read once into registers and written once.
//  * delta_chunk_*       -- a prompt in chunks of 64 tokens.  With b the running sum of log g inside
//    a chunk and S the state before it, the updates of a chunk solve the unit triangular system
//      u_i + beta_i sum_{j<i} e^(b_i - b_j) (k_i.k_j) u_j = beta_i (v_i - e^(b_i) S^T k_i),
//    so U = U0 - W S with U0 = T diag(beta) V, W = T diag(beta e^b) K, T the inverse of the system,
//    none of which needs S: one launch forms them for all chunks at once, a second walks the chunks
//    of a sequence with four float32 matrix products each.  Every exponent is <= 0.
//  * delta_scan_kernel   -- token by token, any size.
#include <algorithm>

#include "lm_launch.h"

namespace lsh {

namespace {

// ------------------------------------------------------------------------------------------------
// Convolution, silu, unit vectors and gates of a prompt.  One wavefront takes one head of q, k or v
// (or the gates) over a tile of tokens and keeps the convolution's window in registers.
constexpr int kConvTile = 16;

template <typename T, int NT>  // at most NT taps
__global__ void __launch_bounds__(256)
delta_prepare_kernel(const T* __restrict__ proj, long ld, const float* __restrict__ ba,
                     const float* __restrict__ conv_w, const float* __restrict__ a_log,
                     const float* __restrict__ dt_bias, const T* __restrict__ ring,
                     float* __restrict__ q, float* __restrict__ k, T* __restrict__ v,
                     float* __restrict__ log_g, float* __restrict__ beta,
                     const SeqSpan* __restrict__ seqs, DeltaShape sh) {
  const SeqSpan sq = seqs[blockIdx.z];
  const int t0 = blockIdx.x * kConvTile;
  if (t0 >= sq.n) return;
  const int t1 = min(t0 + kConvTile, sq.n);
  const int unit = blockIdx.y * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  const int G = sh.kv_heads, H = sh.heads, D = sh.dim, VD = sh.vdim;
  if (unit > 2 * G + H) return;
  if (unit == 2 * G + H) {
    for (int x = lane; x < (t1 - t0) * H; x += 64) {
      const int t = x / H, h = x - t * H;
      const long row = sq.row0 + t0 + t;
      const float b = ba[row * 2 * H + h], a = ba[row * 2 * H + H + h];
      beta[row * H + h] = sigmoid_f(b);
      log_g[row * H + h] = -expf(a_log[h]) * softplus_f(a + dt_bias[h]);
    }
    return;
  }
  const bool is_v = unit >= 2 * G;
  const int n = is_v ? VD : D;
  const int ch0 = is_v ? 2 * G * D + (unit - 2 * G) * VD : unit * D;  // first channel
  const int C = sh.channels();
  float w[NT][2][2], x[NT][2][2];  // [tap][half][pair element]; window: x[NT - 1] is the current token
  auto load = [&](int t, float (&o)[2][2]) {
    const int p = sq.pos0 + t;
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        const int d = 2 * (i * 64 + lane) + e;
        float val = 0.f;
        if (d < n && p >= 0)
          val = t >= 0 ? to_f(proj[(sq.row0 + t) * ld + ch0 + d])
                       : to_f(ring[((long)sq.slot * sh.taps + p % sh.taps) * C + ch0 + d]);
        o[i][e] = val;
      }
  };
#pragma unroll
  for (int s = 0; s < NT; ++s) {
    const int lag = NT - 1 - s;  // tokens back
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        const int d = 2 * (i * 64 + lane) + e;
        w[s][i][e] = d < n && lag < sh.taps ? conv_w[(long)(ch0 + d) * sh.taps + sh.taps - 1 - lag] : 0.f;
        x[s][i][e] = 0.f;
      }
    if (lag > 0 && lag < sh.taps) load(t0 - lag, x[s]);
  }
  float nx[2][2];
  load(t0, nx);
  for (int t = t0; t < t1; ++t) {
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int e = 0; e < 2; ++e) x[NT - 1][i][e] = nx[i][e];
    if (t + 1 < t1) load(t + 1, nx);
    float y[2][2], ss = 0.f;
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        float c = 0.f;
#pragma unroll
        for (int s = 0; s < NT; ++s) c = fmaf(w[s][i][e], x[s][i][e], c);
        y[i][e] = silu_f(c);
        ss += y[i][e] * y[i][e];
      }
    const long row = sq.row0 + t;
    if (is_v) {
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int e = 0; e < 2; ++e) {
          const int d = 2 * (i * 64 + lane) + e;
          if (d < n) v[row * H * VD + (unit - 2 * G) * VD + d] = from_f<T>(y[i][e]);
        }
    } else {
      const bool is_q = unit < G;
      float r = 1.0f / sqrtf(wave_sum_dpp(ss) + 1e-6f);
      if (is_q) r *= 1.0f / sqrtf((float)D);
      float* o = (is_q ? q + (row * G + unit) * D : k + (row * G + unit - G) * D);
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int e = 0; e < 2; ++e) {
          const int d = 2 * (i * 64 + lane) + e;
          if (d < n) o[d] = y[i][e] * r;
        }
    }
#pragma unroll
    for (int s = 0; s < NT - 1; ++s)
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int e = 0; e < 2; ++e) x[s][i][e] = x[s + 1][i][e];
  }
}

// The same for head sizes, columns and row lengths in fours: LPH lanes per head, four channels per
// lane, 64 / LPH heads per wavefront.  The last block row computes the gates.
template <typename T, int NT, int LPH>
__global__ void __launch_bounds__(256)
delta_prepare4_kernel(const T* __restrict__ proj, long ld, const float* __restrict__ ba,
                      const float* __restrict__ conv_w, const float* __restrict__ a_log,
                      const float* __restrict__ dt_bias, const T* __restrict__ ring,
                      float* __restrict__ q, float* __restrict__ k, T* __restrict__ v,
                      float* __restrict__ log_g, float* __restrict__ beta,
                      const SeqSpan* __restrict__ seqs, DeltaShape sh) {
  const SeqSpan sq = seqs[blockIdx.z];
  const int t0 = blockIdx.x * kConvTile;
  if (t0 >= sq.n) return;
  const int t1 = min(t0 + kConvTile, sq.n);
  const int G = sh.kv_heads, H = sh.heads, D = sh.dim, VD = sh.vdim;
  if (blockIdx.y == gridDim.y - 1) {
    for (int x = threadIdx.x; x < (t1 - t0) * H; x += 256) {
      const int t = x / H, h = x - t * H;
      const long row = sq.row0 + t0 + t;
      const float b = ba[row * 2 * H + h], a = ba[row * 2 * H + H + h];
      beta[row * H + h] = sigmoid_f(b);
      log_g[row * H + h] = -expf(a_log[h]) * softplus_f(a + dt_bias[h]);
    }
    return;
  }
  const int unit_raw = (int)(blockIdx.y * 256 + threadIdx.x) / LPH;
  const int unit = min(unit_raw, 2 * G + H - 1);
  const bool is_v = unit >= 2 * G;
  const int n = is_v ? VD : D, d = (threadIdx.x % LPH) * 4;
  const int ch = (is_v ? 2 * G * D + (unit - 2 * G) * VD : unit * D) + d;  // first of four channels
  const bool in = unit_raw < 2 * G + H && d < n;
  const int C = sh.channels();
  float w[NT][4], x[NT][4];  // window: x[NT - 1] is the current token
  auto load = [&](int t, float (&o)[4]) {
    const int p = sq.pos0 + t;
#pragma unroll
    for (int e = 0; e < 4; ++e) o[e] = 0.f;
    if (in && p >= 0) {
      if (t >= 0) ldv<4, T>(proj + (sq.row0 + t) * ld + ch, o);
      else ldv<4, T>(ring + ((long)sq.slot * sh.taps + p % sh.taps) * C + ch, o);
    }
  };
#pragma unroll
  for (int s = 0; s < NT; ++s) {
    const int lag = NT - 1 - s;  // tokens back
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      w[s][e] = in && lag < sh.taps ? conv_w[(long)(ch + e) * sh.taps + sh.taps - 1 - lag] : 0.f;
      x[s][e] = 0.f;
    }
    if (lag > 0 && lag < sh.taps) load(t0 - lag, x[s]);
  }
  float nx[2][4];
  load(t0, nx[0]);
  if (t0 + 1 < t1) load(t0 + 1, nx[1]);
  for (int t = t0; t < t1; ++t) {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      x[NT - 1][e] = nx[0][e];
      nx[0][e] = nx[1][e];
    }
    if (t + 2 < t1) load(t + 2, nx[1]);
    float y[4], ss = 0.f;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      float c = 0.f;
#pragma unroll
      for (int s = 0; s < NT; ++s) c = fmaf(w[s][e], x[s][e], c);
      y[e] = silu_f(c);
      ss += y[e] * y[e];
    }
    ss += dpp_f<kDppXor1>(ss);
    ss += dpp_f<kDppXor2>(ss);
    ss += dpp_f<kDppHalfMirror>(ss);
    ss += dpp_f<kDppMirror>(ss);
    if (LPH > 16) ss += __shfl_xor(ss, 16);
    if (LPH > 32) ss += __shfl_xor(ss, 32);
    const long row = sq.row0 + t;
    if (in) {
      if (is_v) {
        stv<4, T>(v + row * H * VD + (unit - 2 * G) * VD + d, y);
      } else {
        const bool is_q = unit < G;
        float r = 1.0f / sqrtf(ss + 1e-6f);
        if (is_q) r *= 1.0f / sqrtf((float)D);
#pragma unroll
        for (int e = 0; e < 4; ++e) y[e] *= r;
        stv<4, float>((is_q ? q + (row * G + unit) * D : k + (row * G + unit - G) * D) + d, y);
      }
    }
#pragma unroll
    for (int s = 0; s < NT - 1; ++s)
#pragma unroll
      for (int e = 0; e < 4; ++e) x[s][e] = x[s + 1][e];
  }
}

// inputs of the span's last taps positions into the ring (its older readers have finished: stream order)
template <typename T>
__global__ void __launch_bounds__(256)
delta_ring_kernel(const T* __restrict__ proj, long ld, T* __restrict__ ring,
                  const SeqSpan* __restrict__ seqs, DeltaShape sh) {
  const SeqSpan sq = seqs[blockIdx.y];
  const int C = sh.channels();
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= C) return;
  for (int t = max(0, sq.n - sh.taps); t < sq.n; ++t)
    ring[((long)sq.slot * sh.taps + (sq.pos0 + t) % sh.taps) * C + c] = proj[(sq.row0 + t) * ld + c];
}

// ------------------------------------------------------------------------------------------------
// Token by token.  A wavefront owns 4 columns of a head's state, 16 lanes per column, each lane every
// 16th row.
template <typename T>
__global__ void __launch_bounds__(256)
delta_scan_kernel(const float* __restrict__ q, const float* __restrict__ k, const T* __restrict__ v,
                  const float* __restrict__ log_g, const float* __restrict__ beta,
                  float* __restrict__ state, float* __restrict__ o,
                  const SeqSpan* __restrict__ seqs, DeltaShape sh) {
  const SeqSpan sq = seqs[blockIdx.z];
  const int h = blockIdx.y, H = sh.heads, D = sh.dim, VD = sh.vdim, G = sh.kv_heads;
  const int lane = threadIdx.x & 63, rg = lane >> 2;
  const int c = (blockIdx.x * 4 + (threadIdx.x >> 6)) * 4 + (lane & 3);
  const int cc = min(c, VD - 1), kvh = h / (H / G);
  float* sp = state + (((long)sq.slot * H + h) * D) * VD + cc;
  float S[16];
#pragma unroll
  for (int i = 0; i < 16; ++i) {
    const int r = rg + 16 * i;
    S[i] = sq.pos0 > 0 && r < D ? sp[(long)r * VD] : 0.f;
  }
  for (int t = 0; t < sq.n; ++t) {
    const long row = sq.row0 + t;
    const float g = expf(log_g[row * H + h]), b = beta[row * H + h];
    const float vv = to_f(v[(row * H + h) * VD + cc]);
    const float *kr = k + (row * G + kvh) * D, *qr = q + (row * G + kvh) * D;
    float kk[16], p = 0.f;
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int r = rg + 16 * i;
      kk[i] = r < D ? kr[r] : 0.f;
      S[i] *= g;
      p = fmaf(kk[i], S[i], p);
    }
#pragma unroll
    for (int d = 4; d < 64; d <<= 1) p += __shfl_xor(p, d);
    const float u = b * (vv - p);
    float out = 0.f;
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int r = rg + 16 * i;
      S[i] = fmaf(kk[i], u, S[i]);
      out = fmaf(r < D ? qr[r] : 0.f, S[i], out);
    }
#pragma unroll
    for (int d = 4; d < 64; d <<= 1) out += __shfl_xor(out, d);
    if (rg == 0 && c < VD) o[(row * H + h) * VD + c] = out;
  }
  if (c < VD) {
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int r = rg + 16 * i;
      if (r < D) sp[(long)r * VD] = S[i];
    }
  }
}

// ------------------------------------------------------------------------------------------------
// Chunks of 64.  Workspace of one (chunk, head): W [64][D], P [64][64] (decayed q.k, lower triangle),
// U0 [64][VD], b [64].  A sequence's chunk c is number row0 / 64 + sequence index + c.
constexpr int kC = 64;

__host__ __device__ inline long chunk_floats(const DeltaShape& sh) {
  return (long)kC * (sh.dim + kC + sh.vdim + 1);
}

__device__ __forceinline__ frag_t fz() { return (frag_t)0u; }
__device__ __forceinline__ frag_t scale4(frag_t a, const float* s) {
  f32x4 x = __builtin_bit_cast(f32x4, a);
#pragma unroll
  for (int j = 0; j < 4; ++j) x[j] *= s[j];
  return __builtin_bit_cast(frag_t, x);
}

template <typename T, int NDW>  // dim, vdim <= 64 * NDW
__global__ void __launch_bounds__(256)
delta_chunk_prep_kernel(const float* __restrict__ q, const float* __restrict__ k,
                        const T* __restrict__ v, const float* __restrict__ log_g,
                        const float* __restrict__ beta, float* __restrict__ ws,
                        const SeqSpan* __restrict__ seqs, DeltaShape sh) {
  constexpr int LS = kC + 4;
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const SeqSpan sq = seqs[blockIdx.z];
  const int c0 = blockIdx.x * kC;
  if (c0 >= sq.n) return;
  const int n = min(kC, sq.n - c0);
  const int h = blockIdx.y, H = sh.heads, D = sh.dim, VD = sh.vdim, G = sh.kv_heads;
  const int kvh = h / (H / G);
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, c = lane & 15, qd = lane >> 4;
  const int KS = max(D, VD) + 4;  // row stride of the operand region
  float* X = sm;                  // [64][KS]: K, then V
  float* L = X + kC * KS;         // [64][LS]
  float* Tm = L + kC * LS;        // [64][LS]
  float *bs = Tm + kC * LS, *bt = bs + kC, *sc = bt + kC;  // cumulative log g, beta, column scale
  const long row0 = sq.row0 + c0;
  float* out = ws + ((sq.row0 / kC + blockIdx.z + blockIdx.x) * (long)H + h) * chunk_floats(sh);
  float *oW = out, *oP = oW + kC * D, *oU = oP + kC * kC, *ob = oU + kC * VD;
  // everything this chunk reads is requested at once: keys (to LDS), the query fragments of the
  // wavefront's rows, and the values, which wait in registers for their turn in LDS
  typedef T T4 __attribute__((ext_vector_type(4)));
  frag_t kq[4 * NDW], fq[4 * NDW];
  T4 vq[4 * NDW];
  const int qi = w * 16 + c;
  {
    const float* qr = q + ((row0 + min(qi, n - 1)) * G + kvh) * D;
#pragma unroll
    for (int u = 0; u < 4 * NDW; ++u) {
      const int x = u * 256 + tid, r = x / (D / 4), d = (x - r * (D / 4)) * 4;
      kq[u] = r < n ? *reinterpret_cast<const frag_t*>(k + ((row0 + r) * G + kvh) * D + d) : fz();
    }
#pragma unroll
    for (int u = 0; u < 4 * NDW; ++u)
      fq[u] = u < D / 16 && qi < n ? *reinterpret_cast<const frag_t*>(qr + u * 16 + qd * 4) : fz();
#pragma unroll
    for (int u = 0; u < 4 * NDW; ++u) {
      const int x = u * 256 + tid, r = x / (VD / 4), d = (x - r * (VD / 4)) * 4;
      vq[u] = r < n ? *reinterpret_cast<const T4*>(v + ((row0 + r) * H + h) * VD + d) : (T4)0.f;
    }
  }
#pragma unroll
  for (int u = 0; u < 4 * NDW; ++u) {
    const int x = u * 256 + tid, r = x / (D / 4), d = (x - r * (D / 4)) * 4;
    if (r < kC) *reinterpret_cast<frag_t*>(&X[r * KS + d]) = kq[u];
  }
  if (w == 0) {
    float b = lane < n ? log_g[(row0 + lane) * H + h] : 0.f;
#pragma unroll
    for (int d = 1; d < 64; d <<= 1) {
      const float up = __shfl_up(b, d);
      if (lane >= d) b += up;
    }
    const float be = lane < n ? beta[(row0 + lane) * H + h] : 0.f;
    bs[lane] = b;
    bt[lane] = be;
    sc[lane] = be * expf(b);
    ob[lane] = b;
  }
  for (int x = tid; x < kC * LS; x += 256) Tm[x] = 0.f;
  __syncthreads();
  // k_i.k_j and q_i.k_j: wavefront w has the rows 16w .. 16w + 15, column blocks up to its own
  {
    f32x4 kk[4], qk[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) kk[j] = qk[j] = (f32x4)0.f;
#pragma unroll
    for (int s = 0; s < 4 * NDW; ++s)
      if (s < D / 16) {
        const int d = s * 16 + qd * 4;
        const frag_t fk = *reinterpret_cast<const frag_t*>(&X[qi * KS + d]);
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (j <= w) {
            const frag_t fb = *reinterpret_cast<const frag_t*>(&X[(j * 16 + c) * KS + d]);
            kk[j] = mma16(0.f, fk, fb, kk[j]);
            qk[j] = mma16(0.f, fq[s], fb, qk[j]);
          }
      }
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = w * 16 + 4 * qd + r, col = j * 16 + c;
        const float e = col <= i ? expf(bs[i] - bs[col]) : 0.f;
        L[i * LS + col] = col < i ? bt[i] * e * kk[j][r] : 0.f;
        oP[i * kC + col] = e * qk[j][r];
      }
  }
  __syncthreads();
  // inverse of the diagonal blocks of I + L: wavefront w its block, a lane per column
  if (lane < 16) {
    float x[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float s = i == lane ? 1.f : 0.f;
#pragma unroll
      for (int j = 0; j < 16; ++j)
        if (j < i) s = fmaf(-L[(w * 16 + i) * LS + w * 16 + j], x[j], s);
      x[i] = s;
    }
#pragma unroll
    for (int i = 0; i < 16; ++i) Tm[(w * 16 + i) * LS + w * 16 + lane] = x[i];
  }
  __syncthreads();
  // below the diagonal, by distance: T_ij = -T_ii sum_{j <= m < i} L_im T_mj
#pragma unroll
  for (int dist = 1; dist < 4; ++dist) {
    const int r = tid >> 4, cc = tid & 15;
    // rows are read in fours
    auto dot = [&](const float* a, const float* t, int len) {
      float s = 0.f;
      for (int m = 0; m < len; m += 4) {
        const f32x4 x = *reinterpret_cast<const f32x4*>(a + m);
#pragma unroll
        for (int e = 0; e < 4; ++e) s = fmaf(x[e], t[(m + e) * LS], s);
      }
      return s;
    };
    float acc[3];
#pragma unroll
    for (int b = 0; b < 4 - dist; ++b)
      acc[b] = dot(&L[((b + dist) * 16 + r) * LS + b * 16], &Tm[b * 16 * LS + b * 16 + cc], 16 * dist);
    // the sums wait in the target blocks, which nothing else reads at this distance
#pragma unroll
    for (int b = 0; b < 4 - dist; ++b) Tm[((b + dist) * 16 + r) * LS + b * 16 + cc] = acc[b];
    __syncthreads();
#pragma unroll
    for (int b = 0; b < 4 - dist; ++b)
      acc[b] = -dot(&Tm[((b + dist) * 16 + r) * LS + (b + dist) * 16],
                    &Tm[(b + dist) * 16 * LS + b * 16 + cc], 16);
    __syncthreads();
#pragma unroll
    for (int b = 0; b < 4 - dist; ++b) Tm[((b + dist) * 16 + r) * LS + b * 16 + cc] = acc[b];
    __syncthreads();
  }
  // T diag(scale) X for the columns of X, rows of wavefront w
  auto product = [&](const float* scale, float* dst, int cols) {
    frag_t ft[4];
#pragma unroll
    for (int s = 0; s < 4; ++s)
      ft[s] = scale4(*reinterpret_cast<const frag_t*>(&Tm[(w * 16 + c) * LS + s * 16 + qd * 4]),
                     scale + s * 16 + qd * 4);
    for (int cb = 0; cb < cols / 16; ++cb) {
      f32x4 acc = (f32x4)0.f;
#pragma unroll
      for (int s = 0; s < 4; ++s)
        if (s <= w) {
          f32x4 x;
#pragma unroll
          for (int j = 0; j < 4; ++j) x[j] = X[(s * 16 + qd * 4 + j) * KS + cb * 16 + c];
          acc = mma16(0.f, ft[s], __builtin_bit_cast(frag_t, x), acc);
        }
#pragma unroll
      for (int r = 0; r < 4; ++r) dst[(long)(w * 16 + 4 * qd + r) * cols + cb * 16 + c] = acc[r];
    }
  };
  product(sc, oW, D);
  __syncthreads();
#pragma unroll
  for (int u = 0; u < 4 * NDW; ++u) {
    const int x = u * 256 + tid, r = x / (VD / 4), d = (x - r * (VD / 4)) * 4;
    if (r < kC) {
      const f32x4 t = {to_f((T)vq[u][0]), to_f((T)vq[u][1]), to_f((T)vq[u][2]), to_f((T)vq[u][3])};
      *reinterpret_cast<f32x4*>(&X[r * KS + d]) = t;
    }
  }
  __syncthreads();
  product(bt, oU, VD);
}

// One workgroup walks the chunks of one (sequence, head) for 16 * NVB value columns.  The state lies
// in registers as the accumulators of its update (wavefront w: row blocks w, w + 4, ..) and
// transposed in LDS as an operand; the chunk's operands go from global memory straight into
// fragments, each element to the one wavefront that needs it.
template <int NDW, int NVB>  // dim <= 64 * NDW
__global__ void __launch_bounds__(256, NDW == 1 ? 2 : 1)
delta_chunk_scan_kernel(const float* __restrict__ q, const float* __restrict__ k,
                        const float* __restrict__ ws, float* __restrict__ state,
                        float* __restrict__ o, const SeqSpan* __restrict__ seqs, int vblocks,
                        DeltaShape sh) {
  constexpr int MAXD = 64 * NDW, SS = MAXD + 4, US = kC + 4, NS = 4 * NDW;
  extern __shared__ __attribute__((aligned(16))) float sm[];
  float(*St)[SS] = reinterpret_cast<float(*)[SS]>(sm);
  float(*Ut)[US] = reinterpret_cast<float(*)[US]>(sm + NVB * 16 * SS);
  float(*Ud)[US] = Ut + NVB * 16;
  const int H = sh.heads, D = sh.dim, VD = sh.vdim, G = sh.kv_heads;
  // the value blocks of a head read the same operands: H * sequences apart in the grid
  const int hs = gridDim.x / vblocks;
  const int vb = blockIdx.x / hs, rest = blockIdx.x - vb * hs;
  const int si = rest / H, h = rest - si * H;
  const SeqSpan sq = seqs[si];
  const int kvh = h / (H / G);
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, c = lane & 15, qd = lane >> 4;
  const int v0 = vb * NVB * 16, ns = D / 16;
  float* sp = state + ((long)sq.slot * H + h) * D * VD;
  f32x4 S[NDW][NVB];
#pragma unroll
  for (int i = 0; i < NDW; ++i)
#pragma unroll
    for (int b = 0; b < NVB; ++b) {
      const int db = w + 4 * i, vc = v0 + b * 16 + c;
#pragma unroll
      for (int r = 0; r < 4; ++r)
        S[i][b][r] = sq.pos0 > 0 && db < ns && vc < VD
                         ? sp[(long)(db * 16 + 4 * qd + r) * VD + vc] : 0.f;
      if (db < ns)
        *reinterpret_cast<f32x4*>(&St[b * 16 + c][db * 16 + 4 * qd]) = S[i][b];
    }
  const int chunks = (sq.n + kC - 1) / kC;
  const long cf = chunk_floats(sh);
  const float* base = ws + ((sq.row0 / kC + si) * (long)H + h) * cf;
  // The chunk's operands: those of its first half (products with S) and of its second (products with
  // U).  Both are requested at its start; holding a chunk's set ahead costs more in register moves
  // than it hides.
  frag_t fw[NS], fq[NS], fp[4];
  f32x4 fk[NDW][4], u0[NVB], b4;  // b4: cumulative log decay of the rows 4 qd ..
  float b_last;
  auto fetch1 = [&](int ch) {
    const float* pW = base + (long)ch * H * cf;
    const float *pU = pW + kC * (D + kC), *pb = pU + kC * VD;
    const int n = min(kC, sq.n - ch * kC), i = w * 16 + c;
    const float* qr = q + ((sq.row0 + (long)ch * kC + min(i, n - 1)) * G + kvh) * D;
#pragma unroll
    for (int s = 0; s < NS; ++s)
      if (s < ns) {
        fw[s] = *reinterpret_cast<const frag_t*>(pW + (long)i * D + s * 16 + qd * 4);
        fq[s] = *reinterpret_cast<const frag_t*>(qr + s * 16 + qd * 4);
      }
#pragma unroll
    for (int b = 0; b < NVB; ++b)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int vc = v0 + b * 16 + c;
        u0[b][r] = vc < VD ? pU[(long)(w * 16 + 4 * qd + r) * VD + vc] : 0.f;
      }
    b4 = *reinterpret_cast<const f32x4*>(pb + w * 16 + 4 * qd);
    b_last = pb[kC - 1];
  };
  auto fetch2 = [&](int ch) {
    const float* pP = base + (long)ch * H * cf + kC * D;
    const int n = min(kC, sq.n - ch * kC);
    const long row0 = sq.row0 + (long)ch * kC;
#pragma unroll
    for (int s = 0; s < 4; ++s)
      fp[s] = *reinterpret_cast<const frag_t*>(pP + (w * 16 + c) * kC + s * 16 + qd * 4);
#pragma unroll
    for (int x = 0; x < NDW; ++x) {
      const int db = w + 4 * x;
#pragma unroll
      for (int s = 0; s < 4; ++s)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int t = s * 16 + qd * 4 + j;
          fk[x][s][j] = db < ns && t < n ? k[((row0 + t) * G + kvh) * D + db * 16 + c] : 0.f;
        }
    }
  };
  __syncthreads();
  for (int ch = 0; ch < chunks; ++ch) {
    fetch1(ch);
    fetch2(ch);
    const int n = min(kC, sq.n - ch * kC);
    f32x4 ws_acc[NVB], o_acc[NVB];
#pragma unroll
    for (int b = 0; b < NVB; ++b) ws_acc[b] = o_acc[b] = (f32x4)0.f;
#pragma unroll
    for (int s = 0; s < NS; ++s)
      if (s < ns) {
#pragma unroll
        for (int b = 0; b < NVB; ++b) {
          const frag_t fs = *reinterpret_cast<const frag_t*>(&St[b * 16 + c][s * 16 + qd * 4]);
          ws_acc[b] = mma16(0.f, fw[s], fs, ws_acc[b]);
          o_acc[b] = mma16(0.f, fq[s], fs, o_acc[b]);
        }
      }
    f32x4 e_row, e_left;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      e_row[r] = expf(b4[r]);
      e_left[r] = expf(b_last - b4[r]);
    }
    const float decay = expf(b_last);
#pragma unroll
    for (int b = 0; b < NVB; ++b) {
      const f32x4 u = u0[b] - ws_acc[b];
      o_acc[b] *= e_row;
      *reinterpret_cast<f32x4*>(&Ut[b * 16 + c][w * 16 + 4 * qd]) = u;
      *reinterpret_cast<f32x4*>(&Ud[b * 16 + c][w * 16 + 4 * qd]) = u * e_left;
    }
    __syncthreads();
#pragma unroll
    for (int b = 0; b < NVB; ++b) {
#pragma unroll
      for (int s = 0; s < 4; ++s)
        if (s <= w)
          o_acc[b] = mma16(0.f, fp[s],
                           *reinterpret_cast<const frag_t*>(&Ut[b * 16 + c][s * 16 + qd * 4]),
                           o_acc[b]);
#pragma unroll
      for (int x = 0; x < NDW; ++x) {
        const int db = w + 4 * x;
        if (db < ns) {
          S[x][b] *= decay;
#pragma unroll
          for (int s = 0; s < 4; ++s)
            S[x][b] = mma16(0.f, __builtin_bit_cast(frag_t, fk[x][s]),
                            *reinterpret_cast<const frag_t*>(&Ud[b * 16 + c][s * 16 + qd * 4]),
                            S[x][b]);
          *reinterpret_cast<f32x4*>(&St[b * 16 + c][db * 16 + 4 * qd]) = S[x][b];
        }
      }
    }
#pragma unroll
    for (int b = 0; b < NVB; ++b)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = w * 16 + 4 * qd + r, vc = v0 + b * 16 + c;
        if (t < n && vc < VD)
          o[((sq.row0 + (long)ch * kC + t) * H + h) * VD + vc] = o_acc[b][r];
      }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < NDW; ++i)
#pragma unroll
    for (int b = 0; b < NVB; ++b) {
      const int db = w + 4 * i, vc = v0 + b * 16 + c;
      if (db < ns && vc < VD) {
#pragma unroll
        for (int r = 0; r < 4; ++r) sp[(long)(db * 16 + 4 * qd + r) * VD + vc] = S[i][b][r];
      }
    }
}

// ------------------------------------------------------------------------------------------------
template <typename T>
__global__ void __launch_bounds__(256)
delta_gated_norm_kernel(const float* __restrict__ o, const T* __restrict__ proj, long ld, int g_col,
                        const float* __restrict__ norm_w, float eps, T* __restrict__ out,
                        long units, DeltaShape sh) {
  const long unit = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (unit >= units) return;
  const int lane = threadIdx.x & 63, VD = sh.vdim;
  const long row = unit / sh.heads;
  const int h = (int)(unit - row * sh.heads);
  const float* src = o + unit * VD;
  float x[2][2], ss = 0.f;
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int e = 0; e < 2; ++e) {
      const int d = 2 * (i * 64 + lane) + e;
      x[i][e] = d < VD ? src[d] : 0.f;
      ss += x[i][e] * x[i][e];
    }
  const float r = 1.0f / sqrtf(wave_sum_dpp(ss) / (float)VD + eps);
  const T* gate = proj + row * ld + g_col + h * VD;
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int e = 0; e < 2; ++e) {
      const int d = 2 * (i * 64 + lane) + e;
      if (d < VD) out[unit * VD + d] = from_f<T>(x[i][e] * r * norm_w[d] * silu_f(to_f(gate[d])));
    }
}

// LPH lanes per head, four elements per lane
template <typename T, int LPH>
__global__ void __launch_bounds__(256)
delta_gated_norm4_kernel(const float* __restrict__ o, const T* __restrict__ proj, long ld, int g_col,
                         const float* __restrict__ norm_w, float eps, T* __restrict__ out, int units,
                         DeltaShape sh) {
  const int unit_raw = (int)((blockIdx.x * 256 + threadIdx.x) / LPH);
  const int unit = min(unit_raw, units - 1), VD = sh.vdim, d = (threadIdx.x % LPH) * 4;
  const int row = unit / sh.heads, h = unit - row * sh.heads;
  float x[4] = {0.f, 0.f, 0.f, 0.f}, z[4], w[4];
  const bool in = d < VD;
  if (in) {
    ldv<4, float>(o + (long)unit * VD + d, x);
    ldv<4, T>(proj + row * ld + g_col + h * VD + d, z);
    ldv<4, float>(norm_w + d, w);
  }
  float ss = x[0] * x[0] + x[1] * x[1] + x[2] * x[2] + x[3] * x[3];
  ss += dpp_f<kDppXor1>(ss);
  ss += dpp_f<kDppXor2>(ss);
  ss += dpp_f<kDppHalfMirror>(ss);
  ss += dpp_f<kDppMirror>(ss);
  if (LPH > 16) ss += __shfl_xor(ss, 16);
  if (LPH > 32) ss += __shfl_xor(ss, 32);
  const float r = 1.0f / sqrtf(ss / (float)VD + eps);
  if (in && unit_raw < units) {
#pragma unroll
    for (int e = 0; e < 4; ++e) x[e] = x[e] * r * w[e] * silu_f(z[e]);
    stv<4, T>(out + (long)unit * VD + d, x);
  }
}

// ------------------------------------------------------------------------------------------------
// One token.  Workgroup per (row, head).  Threads form column groups of V value columns times row
// groups; a thread holds rows rg, rg + nrg, .. (at most RM) of its V columns.
template <typename T, int V, int RM, int NTH>
__global__ void __launch_bounds__(NTH)
delta_step_kernel(const T* __restrict__ proj, long ld, int g_col, const float* __restrict__ ba,
                  const float* __restrict__ conv_w, const float* __restrict__ a_log,
                  const float* __restrict__ dt_bias, const float* __restrict__ norm_w, float eps,
                  T* __restrict__ ring, float* __restrict__ state, T* __restrict__ out,
                  const int* __restrict__ row_slot, const int* __restrict__ row_pos, int nrg,
                  DeltaShape sh) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  __shared__ float red[4][16];
  const int H = sh.heads, D = sh.dim, VD = sh.vdim, G = sh.kv_heads, C = sh.channels();
  float *qs = sm, *ks = qs + D, *vs = ks + D, *part = vs + VD;  // part [2][nrg][VD]
  const long row = blockIdx.x;
  const int h = blockIdx.y, rep = H / G, kvh = h / rep;
  const int tid = threadIdx.x, slot = row_slot[row], pos = row_pos[row];
  const int ncg = (VD + V - 1) / V;
  const int rg = tid / ncg, c = (tid - rg * ncg) * V;
  const bool act = rg < nrg;
  float* sp = state + ((long)slot * H + h) * D * VD + c;
  float S[RM][V];
#pragma unroll
  for (int i = 0; i < RM; ++i) {
    const int r = rg + nrg * i;
    if (act && r < D && pos > 0) {
      ldv<V, float>(sp + (long)r * VD, S[i]);
    } else {
#pragma unroll
      for (int e = 0; e < V; ++e) S[i][e] = 0.f;
    }
  }
  const float be = sigmoid_f(ba[row * 2 * H + h]);
  const float g = expf(-expf(a_log[h]) * softplus_f(ba[row * 2 * H + H + h] + dt_bias[h]));
  float sq_q = 0.f, sq_k = 0.f;
  for (int x = tid; x < 2 * D + VD; x += NTH) {
    const int ch = x < D ? kvh * D + x : x < 2 * D ? (G + kvh) * D + x - D
                                                   : 2 * G * D + h * VD + x - 2 * D;
    const T cur = proj[row * ld + ch];
    float y = conv_w[(long)ch * sh.taps + sh.taps - 1] * to_f(cur);
    for (int lag = 1; lag < sh.taps; ++lag)
      if (pos - lag >= 0)
        y = fmaf(conv_w[(long)ch * sh.taps + sh.taps - 1 - lag],
                 to_f(ring[((long)slot * sh.taps + (pos - lag) % sh.taps) * C + ch]), y);
    y = silu_f(y);
    qs[x] = y;  // q, k, v lie one after the other
    if (x < D) sq_q += y * y;
    else if (x < 2 * D) sq_k += y * y;
    // the entry written is not among those any head reads for this position
    if (x >= 2 * D || h % rep == 0)
      ring[((long)slot * sh.taps + pos % sh.taps) * C + ch] = cur;
  }
  sq_q = block_sum_dpp(sq_q, red[0]);
  sq_k = block_sum_dpp(sq_k, red[1]);
  const float rq = 1.0f / sqrtf(sq_q + 1e-6f) / sqrtf((float)D), rk = 1.0f / sqrtf(sq_k + 1e-6f);
  float pk[V], pq[V];
#pragma unroll
  for (int e = 0; e < V; ++e) pk[e] = pq[e] = 0.f;
#pragma unroll
  for (int i = 0; i < RM; ++i) {
    const int r = rg + nrg * i;
    if (act && r < D) {
      const float kr = ks[r] * rk, qr = qs[r] * rq;
#pragma unroll
      for (int e = 0; e < V; ++e) {
        S[i][e] *= g;
        pk[e] = fmaf(kr, S[i][e], pk[e]);
        pq[e] = fmaf(qr, S[i][e], pq[e]);
      }
    }
  }
  if (act) {
#pragma unroll
    for (int e = 0; e < V; ++e) {
      part[rg * VD + c + e] = pk[e];
      part[(nrg + rg) * VD + c + e] = pq[e];
    }
  }
  float dot = 0.f;
  for (int d = tid; d < D; d += NTH) dot += (qs[d] * rq) * (ks[d] * rk);
  dot = block_sum_dpp(dot, red[2]);  // its barrier also publishes `part`
  // column sums; the update takes the place of v
  float o_c = 0.f;
  for (int x = tid; x < VD; x += NTH) {
    float a = 0.f, b = 0.f;
    for (int i = 0; i < nrg; ++i) {
      a += part[i * VD + x];
      b += part[(nrg + i) * VD + x];
    }
    const float u = be * (vs[x] - a);
    vs[x] = u;
    o_c = fmaf(dot, u, b);  // S^T q after the write: the decayed state's share plus (q.k) u
  }
  const float rms = block_sum_dpp(tid < VD ? o_c * o_c : 0.f, red[3]);
  if (tid < VD) {
    const float r = 1.0f / sqrtf(rms / (float)VD + eps);
    const float z = to_f(proj[row * ld + g_col + h * VD + tid]);
    out[(row * H + h) * VD + tid] = from_f<T>(o_c * r * norm_w[tid] * silu_f(z));
  }
  if (act) {
    float u[V];
#pragma unroll
    for (int e = 0; e < V; ++e) u[e] = vs[c + e];
#pragma unroll
    for (int i = 0; i < RM; ++i) {
      const int r = rg + nrg * i;
      if (r < D) {
        const float kr = ks[r] * rk;
#pragma unroll
        for (int e = 0; e < V; ++e) S[i][e] = fmaf(kr, u[e], S[i][e]);
        stv<V, float>(sp + (long)r * VD, S[i]);
      }
    }
  }
}

int check_shape(const DeltaShape& sh) {
  if (sh.heads <= 0 || sh.kv_heads <= 0 || sh.heads % sh.kv_heads != 0 || sh.dim <= 0 ||
      sh.vdim <= 0 || sh.taps <= 0)
    return lsh_fail(LSH_ERR_INVALID, "delta: bad shape");
  if (sh.dim > 256 || sh.vdim > 256 || sh.taps > 16)
    return lsh_fail(LSH_ERR_UNSUPPORTED, "delta: head sizes up to 256, at most 16 taps");
  return LSH_OK;
}

}  // namespace

template <typename T>
int delta_prepare(const T* proj, long ld, const float* ba, const float* conv_w, const float* a_log,
                  const float* dt_bias, T* conv_ring, float* q, float* k, T* v, float* log_g,
                  float* beta, const SeqSpan* seqs, int n_seqs, int max_n, const DeltaShape& sh,
                  hipStream_t s) {
  if (int rc = check_shape(sh)) return rc;
  if (!proj || !ba || !conv_w || !a_log || !dt_bias || !conv_ring || !q || !k || !v || !log_g ||
      !beta || !seqs || n_seqs <= 0 || max_n <= 0 || n_seqs > 65535)
    return lsh_fail(LSH_ERR_INVALID, "delta_prepare: bad arguments");
  const int tiles = (max_n + kConvTile - 1) / kConvTile, units = 2 * sh.kv_heads + sh.heads;
  const dim3 grid(tiles, (units + 1 + 3) / 4, n_seqs);
  if (sh.dim % 4 == 0 && sh.vdim % 4 == 0 && ld % 4 == 0 && sh.taps <= 8) {
    const int wide = std::max(sh.dim, sh.vdim);
#define PREP4(NT, LPH)                                                                             \
  delta_prepare4_kernel<T, NT, LPH><<<dim3(tiles, (units * LPH + 255) / 256 + 1, n_seqs), 256, 0,  \
                                      s>>>(proj, ld, ba, conv_w, a_log, dt_bias, conv_ring, q, k,  \
                                           v, log_g, beta, seqs, sh)
#define PREP4_T(LPH)                  \
  do {                                \
    if (sh.taps <= 4) PREP4(4, LPH);  \
    else PREP4(8, LPH);               \
  } while (0)
    if (wide <= 64) PREP4_T(16);
    else if (wide <= 128) PREP4_T(32);
    else PREP4_T(64);
#undef PREP4_T
#undef PREP4
  } else if (sh.taps <= 4) {
    delta_prepare_kernel<T, 4><<<grid, 256, 0, s>>>(proj, ld, ba, conv_w, a_log, dt_bias, conv_ring,
                                                    q, k, v, log_g, beta, seqs, sh);
  } else {
    delta_prepare_kernel<T, 16><<<grid, 256, 0, s>>>(proj, ld, ba, conv_w, a_log, dt_bias, conv_ring,
                                                    q, k, v, log_g, beta, seqs, sh);
  }
  if (int rc = lsh_check_launch("delta_prepare_kernel")) return rc;
  delta_ring_kernel<T><<<dim3((sh.channels() + 255) / 256, n_seqs), 256, 0, s>>>(proj, ld, conv_ring,
                                                                                seqs, sh);
  return lsh_check_launch("delta_ring_kernel");
}

template <typename T>
int delta_scan(const float* q, const float* k, const T* v, const float* log_g, const float* beta,
               float* state, float* o, const SeqSpan* seqs, int n_seqs, const DeltaShape& sh,
               hipStream_t s) {
  if (int rc = check_shape(sh)) return rc;
  if (!q || !k || !v || !log_g || !beta || !state || !o || !seqs || n_seqs <= 0 || n_seqs > 65535)
    return lsh_fail(LSH_ERR_INVALID, "delta_scan: bad arguments");
  delta_scan_kernel<T><<<dim3((sh.vdim + 15) / 16, sh.heads, n_seqs), 256, 0, s>>>(
      q, k, v, log_g, beta, state, o, seqs, sh);
  return lsh_check_launch("delta_scan_kernel");
}

bool delta_chunked_supported(const DeltaShape& sh) {
  return sh.dim % 16 == 0 && sh.vdim % 16 == 0 && sh.dim <= 256 && sh.vdim <= 256;
}

size_t delta_chunked_workspace(int rows, int n_seqs, const DeltaShape& sh) {
  return ((size_t)rows / kC + n_seqs) * sh.heads * chunk_floats(sh);
}

template <typename T>
int delta_chunked(const float* q, const float* k, const T* v, const float* log_g,
                  const float* beta, float* state, float* o, float* workspace,
                  const SeqSpan* seqs, int n_seqs, int max_n, int rows, const DeltaShape& sh,
                  hipStream_t s) {
  if (int rc = check_shape(sh)) return rc;
  if (!q || !k || !v || !log_g || !beta || !state || !o || !workspace || !seqs || n_seqs <= 0 ||
      max_n <= 0 || max_n > rows || n_seqs > 65535)
    return lsh_fail(LSH_ERR_INVALID, "delta_chunked: bad arguments");
  if (!delta_chunked_supported(sh))
    return lsh_fail(LSH_ERR_UNSUPPORTED, "delta_chunked: head sizes must be multiples of 16");
  const int widest = std::max(sh.dim, sh.vdim);
  auto prep = widest <= 64    ? delta_chunk_prep_kernel<T, 1>
              : widest <= 128 ? delta_chunk_prep_kernel<T, 2>
                              : delta_chunk_prep_kernel<T, 4>;
  const size_t smem = sizeof(float) * ((size_t)kC * (std::max(sh.dim, sh.vdim) + 4) +
                                       2 * (size_t)kC * (kC + 4) + 3 * kC);
  if (int rc = lsh_check_hip(hipFuncSetAttribute(reinterpret_cast<const void*>(prep),
                                                 hipFuncAttributeMaxDynamicSharedMemorySize,
                                                 (int)smem),
                             "hipFuncSetAttribute(delta_chunk_prep)"))
    return rc;
  prep<<<dim3((max_n + kC - 1) / kC, sh.heads, n_seqs), 256, smem, s>>>(q, k, v, log_g, beta,
                                                                        workspace, seqs, sh);
  if (int rc = lsh_check_launch("delta_chunk_prep_kernel")) return rc;
  // value columns per workgroup: as many as leave every compute unit one (they share the operands)
  int nvb = sh.dim > 128 ? 2 : 4;
  while (nvb > 1 && (long)sh.heads * n_seqs * ((sh.vdim + 16 * nvb - 1) / (16 * nvb)) < cu_count())
    nvb /= 2;
  const int vblocks = (sh.vdim + 16 * nvb - 1) / (16 * nvb);
  const unsigned grid = (unsigned)vblocks * sh.heads * n_seqs;
#define SCAN(NDW, NVB)                                                                            \
  do {                                                                                            \
    auto scan = delta_chunk_scan_kernel<NDW, NVB>;                                                \
    const int lds = (int)sizeof(float) * NVB * 16 * (64 * NDW + 4 + 2 * (kC + 4));                \
    if (int rc = lsh_check_hip(hipFuncSetAttribute(reinterpret_cast<const void*>(scan),           \
                                                   hipFuncAttributeMaxDynamicSharedMemorySize,    \
                                                   lds),                                          \
                               "hipFuncSetAttribute(delta_chunk_scan)"))                          \
      return rc;                                                                                  \
    scan<<<grid, 256, lds, s>>>(q, k, workspace, state, o, seqs, vblocks, sh);                    \
  } while (0)
#define SCAN_V(NDW)              \
  do {                           \
    if (nvb == 4) SCAN(NDW, 4);  \
    else if (nvb == 2) SCAN(NDW, 2); \
    else SCAN(NDW, 1);           \
  } while (0)
  if (sh.dim <= 64) SCAN_V(1);
  else if (sh.dim <= 128) SCAN_V(2);
  else if (nvb == 2) SCAN(4, 2);
  else SCAN(4, 1);
#undef SCAN_V
#undef SCAN
  return lsh_check_launch("delta_chunk_scan_kernel");
}

template <typename T>
int delta_gated_norm(const float* o, const T* proj, long ld, int g_col, const float* norm_w,
                     float eps, T* out, int rows, const DeltaShape& sh, hipStream_t s) {
  if (int rc = check_shape(sh)) return rc;
  if (!o || !proj || !norm_w || !out || rows <= 0)
    return lsh_fail(LSH_ERR_INVALID, "delta_gated_norm: bad arguments");
  const long units = (long)rows * sh.heads;
  if (sh.vdim % 4 == 0 && ld % 4 == 0 && g_col % 4 == 0 && units < (1L << 24)) {
#define NORM4(LPH)                                                                        \
  delta_gated_norm4_kernel<T, LPH><<<(unsigned)((units * LPH + 255) / 256), 256, 0, s>>>( \
      o, proj, ld, g_col, norm_w, eps, out, (int)units, sh)
    if (sh.vdim <= 64) NORM4(16);
    else if (sh.vdim <= 128) NORM4(32);
    else NORM4(64);
#undef NORM4
    return lsh_check_launch("delta_gated_norm4_kernel");
  }
  delta_gated_norm_kernel<T><<<(unsigned)((units + 3) / 4), 256, 0, s>>>(o, proj, ld, g_col, norm_w,
                                                                        eps, out, units, sh);
  return lsh_check_launch("delta_gated_norm_kernel");
}

template <typename T>
int delta_step(const T* proj, long ld, int g_col, const float* ba, const float* conv_w,
               const float* a_log, const float* dt_bias, const float* norm_w, float eps,
               T* conv_ring, float* state, T* out, const int* row_slot, const int* row_pos,
               int rows, const DeltaShape& sh, hipStream_t s) {
  if (int rc = check_shape(sh)) return rc;
  if (!proj || !ba || !conv_w || !a_log || !dt_bias || !norm_w || !conv_ring || !state || !out ||
      !row_slot || !row_pos || rows <= 0 || sh.heads > 65535)
    return lsh_fail(LSH_ERR_INVALID, "delta_step: bad arguments");
  const int V = sh.vdim % 4 == 0 ? 4 : 1;
  const int ncg = sh.vdim / V, rm = V == 4 ? 16 : 64;
  int nth = 256, nrg = std::min(nth / ncg, sh.dim);
  if (nrg < 1 || (sh.dim + nrg - 1) / nrg > rm) {
    nth = 1024;
    nrg = std::min(nth / ncg, sh.dim);
  }
  const size_t smem = sizeof(float) * (2 * (size_t)sh.dim + sh.vdim + 2 * (size_t)nrg * sh.vdim);
  const dim3 grid(rows, sh.heads);
#define STEP(V, RM, NTH)                                                                          \
  delta_step_kernel<T, V, RM, NTH><<<grid, NTH, smem, s>>>(                                       \
      proj, ld, g_col, ba, conv_w, a_log, dt_bias, norm_w, eps, conv_ring, state, out, row_slot,  \
      row_pos, nrg, sh)
  if (V == 4) {
    if (nth == 1024) STEP(4, 16, 1024);
    else if ((sh.dim + nrg - 1) / nrg <= 4) STEP(4, 4, 256);
    else STEP(4, 16, 256);
  } else {
    if (nth == 1024) STEP(1, 64, 1024);
    else STEP(1, 64, 256);
  }
#undef STEP
  return lsh_check_launch("delta_step_kernel");
}

#define INST(T)                                                                                    \
  template int delta_prepare<T>(const T*, long, const float*, const float*, const float*,          \
                                const float*, T*, float*, float*, T*, float*, float*,              \
                                const SeqSpan*, int, int, const DeltaShape&, hipStream_t);         \
  template int delta_scan<T>(const float*, const float*, const T*, const float*, const float*,     \
                             float*, float*, const SeqSpan*, int, const DeltaShape&, hipStream_t); \
  template int delta_chunked<T>(const float*, const float*, const T*, const float*, const float*,  \
                                float*, float*, float*, const SeqSpan*, int, int, int,             \
                                const DeltaShape&, hipStream_t);                                   \
  template int delta_gated_norm<T>(const float*, const T*, long, int, const float*, float, T*,     \
                                   int, const DeltaShape&, hipStream_t);                           \
  template int delta_step<T>(const T*, long, int, const float*, const float*, const float*,        \
                             const float*, const float*, float, T*, float*, T*, const int*,        \
                             const int*, int, const DeltaShape&, hipStream_t);
INST(float)
INST(bf16_t)

}  // namespace lsh
