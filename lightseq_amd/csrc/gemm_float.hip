// Matrix products of the floating-point decoders:  C[m, n] = sum_k A[m, k] W[n, k], bfloat16 or
// float32 operands, float32 accumulation, plain or over the rows of an expert.
//
//  * gemm_tile_kernel    -- many rows.  The output tile (128 x 128, or smaller when that leaves
//    compute units idle) is cut like the int8 tile of gemm_tile.h: 128-byte K steps brought from
//    L2 straight into XOR-swizzled LDS rows, 32-byte slices as 32 x 32 matrix-core products; two
//    stages and two workgroups per compute unit hide the loads.
//  * gemm_skinny_kernel  -- few rows (decoding).  A workgroup owns 16 output columns; its four
//    wavefronts split K and load fragments from global memory straight into registers, so the
//    weights are read once at full line width.
//  * gemm_generic_kernel -- any size and alignment.
// The expert products use the same kernels with gathered rows: a tile finds its expert from the
// per-expert counts, so nothing is sorted and no row is copied.
#include <algorithm>

#include "lm_launch.h"
#include "tile_common.h"

namespace lsh {

namespace {

enum GemmMode { kDense = 0, kMoeUp = 1, kMoeDown = 2, kGated = 3 };
constexpr bool is_dense(int mode) { return mode == kDense || mode == kGated; }  // all rows, in order
constexpr bool is_up(int mode) { return mode == kMoeUp || mode == kGated; }     // gate and up rows

struct GemmArgs {
  const void *A, *W;
  void* C;
  float* C2;
  long lda, ldc, ld2;
  int n_split;
  int M, N, K;  // kGated: weights [2][N][K]; kMoeUp: N = ff, weights [experts][2][N][K]; kMoeDown: [experts][N][K]
  const int *count, *list;
  int list_stride, experts, top;
  int planes, k_per_plane;  // gemm_skinny_kernel, kDense
  GemmEpilogue epi;         // kDense
  int act;                  // kMoeUp, kGated
  // gemm_skinny_kernel, kDense: a second product of the same M, N and ldc (blockIdx.z == 1)
  struct {
    const void *A, *W;
    void* C;
    long lda;
    int K, planes, k_per_plane;
  } other;
};

// rows of one tile: where they are read and written
struct RowSet {
  int expert, first, last;  // rows [first, last) of the expert's list, or of the matrix
};

__device__ __forceinline__ float gated(const GemmArgs& a, float gate, float up) {
  return (a.act == kGateRelu ? fmaxf(gate, 0.f) : silu_f(gate)) * up;
}
// the result of column n from its sum
template <int MODE>
__device__ __forceinline__ float finish(const GemmArgs& a, int n, float sum) {
  if (MODE != kDense) return sum;
  const float v = sum * a.epi.scale;
  return a.epi.bias ? v + a.epi.bias[n] : v;
}

template <int MODE>
__device__ __forceinline__ long src_row(const GemmArgs& a, const RowSet& rs, int r) {
  r = min(r, rs.last - 1);
  if (is_dense(MODE)) return r;
  const int id = a.list[(long)rs.expert * a.list_stride + r];
  return MODE == kMoeUp ? id / a.top : id;
}
template <int MODE>
__device__ __forceinline__ long dst_row(const GemmArgs& a, const RowSet& rs, int r) {
  return is_dense(MODE) ? r : a.list[(long)rs.expert * a.list_stride + r];
}

// the t-th tile of `tm` rows, the experts' rows one after the other (all lanes call it)
__device__ __forceinline__ bool expert_tile(const GemmArgs& a, int t, int tm, RowSet& rs) {
  const int lane = threadIdx.x & 63;
  int before = 0;
  for (int e0 = 0; e0 < a.experts; e0 += 64) {
    const int cnt = e0 + lane < a.experts ? a.count[e0 + lane] : 0;
    const int tiles = (cnt + tm - 1) / tm;
    int pre = tiles;
#pragma unroll
    for (int d = 1; d < 64; d <<= 1) {
      const int up = __shfl_up(pre, d);
      if (lane >= d) pre += up;
    }
    const unsigned long long hit = __ballot(before + pre > t);
    if (hit) {
      // the same in every lane: readlane keeps it (and the operand bases) in scalar registers
      const int l = __ffsll(hit) - 1;
      const int c = __builtin_amdgcn_readlane(cnt, l), p = __builtin_amdgcn_readlane(pre, l);
      const int tile = t - (before + p - (c + tm - 1) / tm);
      rs = RowSet{e0 + l, tile * tm, min(c, tile * tm + tm)};
      return true;
    }
    before += __builtin_amdgcn_readlane(pre, 63);
  }
  return false;
}

template <typename TO>
__device__ __forceinline__ void store_col(const GemmArgs& a, long row, int n, float v) {
  if (n < a.n_split) reinterpret_cast<TO*>(a.C)[row * a.ldc + n] = from_f<TO>(v);
  else a.C2[row * a.ld2 + (n - a.n_split)] = v;
}

// ------------------------------------------------------------------------------------------------
// tile_of of the int8 products: contiguous runs of tiles per XCD, 8-tile-tall groups
__device__ __forceinline__ void dense_tile(int t, int nblk, int tiles_m, int tiles_n, int& tm,
                                           int& tn) {
  const int per = nblk / 8, rem = nblk % 8;
  const int xcd = t % 8, loc = t / 8;
  const int pid = xcd * per + (xcd < rem ? xcd : rem) + loc;
  const int grp = pid / (8 * tiles_n), in_grp = pid - grp * 8 * tiles_n;
  const int gm = min(tiles_m - grp * 8, 8);
  tn = in_grp / gm;
  tm = grp * 8 + (in_grp - tn * gm);
}

// 4 wavefronts in 2 x 2, each MB x NB blocks of 32 x 32.  kMoeUp and kGated need NB == 2: block column 0 is
// the gate, 1 the up projection of the same 32 outputs, so a lane holds both.
template <typename T, typename TO, int MODE, int MB, int NB>
__global__ void __launch_bounds__(256)
gemm_tile_kernel(GemmArgs a, int tiles_m, int tiles_n) {
  constexpr int TM = 64 * MB, TN = 64 * NB;
  constexpr int OUT_N = is_up(MODE) ? TN / 2 : TN;  // output columns of a tile
  constexpr int STAGE = (TM + TN) * kBK;
  constexpr int NA = TM / 32, NW = TN / 32, PER = NA + NW;
  static_assert(!is_up(MODE) || NB == 2, "gate and up blocks");
  __shared__ __attribute__((aligned(128))) int8_t smem[2 * STAGE];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int wm = wave >> 1, wn = wave & 1, l32 = lane & 31, g = lane >> 5;
  RowSet rs;
  int tn;
  if (is_dense(MODE)) {
    int tm;
    dense_tile(blockIdx.x, gridDim.x, tiles_m, tiles_n, tm, tn);
    rs = RowSet{0, tm * TM, min(a.M, tm * TM + TM)};
  } else {
    // consecutive workgroups walk the columns of one row tile
    tn = blockIdx.x % tiles_n;
    if (!expert_tile(a, blockIdx.x / tiles_n, TM, rs)) return;
  }
  const int n0 = tn * OUT_N;
  const int Kb = a.K * (int)sizeof(T);  // bytes of a row
  const int nk = Kb / kBK;
  const char* A = reinterpret_cast<const char*>(a.A);
  const char* W = reinterpret_cast<const char*>(a.W);
  if (!is_dense(MODE)) W += (long)rs.expert * (is_up(MODE) ? 2 : 1) * a.N * Kb;

  uint32_t a_src[NA], w_src[NW];
#pragma unroll
  for (int i = 0; i < NA; ++i) {
    const int row = (wave + 4 * i) * 8 + (lane >> 3);
    const int c = (lane & 7) ^ key_act(row);
    a_src[i] = (uint32_t)(src_row<MODE>(a, rs, rs.first + row) * a.lda * (long)sizeof(T)) + c * 16;
  }
#pragma unroll
  for (int i = 0; i < NW; ++i) {
    const int row = (wave + 4 * i) * 8 + (lane >> 3);
    const int c = (lane & 7) ^ key_wgt(row);
    int n;
    if (is_up(MODE)) {
      const int blk = row >> 5;  // wn * 2 + (gate | up)
      n = min(n0 + (blk >> 1) * 32 + (row & 31), a.N - 1) + (blk & 1) * a.N;
    } else {
      n = min(n0 + row, a.N - 1);
    }
    w_src[i] = (uint32_t)n * (uint32_t)Kb + c * 16;
  }
  const uint32_t lds0 = (uint32_t)(uintptr_t)((__attribute__((address_space(3))) void*)smem);
  auto dma1 = [&](const char* base, uint32_t voff, uint32_t lds) {
    lds = __builtin_amdgcn_readfirstlane(lds);
    asm volatile("s_mov_b32 m0, %0\n\tglobal_load_lds_dwordx4 %1, %2" ::"s"(lds), "v"(voff),
                 "s"(base)
                 : "memory");
  };
  auto issue = [&](int kt, int slot) {
    const uint32_t base = lds0 + slot * STAGE;
#pragma unroll
    for (int i = 0; i < NA; ++i) dma1(A + kt * kBK, a_src[i], base + (wave + 4 * i) * 1024);
#pragma unroll
    for (int i = 0; i < NW; ++i)
      dma1(W + kt * kBK, w_src[i], base + TM * kBK + (wave + 4 * i) * 1024);
  };
  // float output: activations are the first operand, a store then covers whole lines; otherwise the
  // weights are, and a lane's 16 accumulators are 16 adjacent columns of one row
  constexpr bool ROWS_IN_REGS = sizeof(TO) == 4 && !is_up(MODE);
  int a_base[MB], w_base[NB];
#pragma unroll
  for (int i = 0; i < MB; ++i) {
    const int row = wm * (MB * 32) + i * 32 + l32;
    a_base[i] = row * kBK + ((g ^ key_act(row)) << 4);
  }
#pragma unroll
  for (int j = 0; j < NB; ++j) {
    const int row = wn * (NB * 32) + j * 32 + sigma(l32);
    w_base[j] = TM * kBK + row * kBK + ((g ^ key_wgt(row)) << 4);
  }
  f32x16v acc[MB][NB];
#pragma unroll
  for (int i = 0; i < MB; ++i)
#pragma unroll
    for (int j = 0; j < NB; ++j) acc[i][j] = (f32x16v)0.f;

  issue(0, 0);
  for (int kt = 0; kt < nk; ++kt) {
    if (kt + 1 < nk) {
      issue(kt + 1, (kt + 1) & 1);
      wait_vmcnt<PER>();
    } else {
      wait_vmcnt<0>();
    }
    asm volatile("s_barrier" ::: "memory");
    const int8_t* stage = smem + (kt & 1) * STAGE;
#pragma unroll
    for (int ks = 0; ks < 4; ++ks) {
      frag_t fa[MB], fw[NB];
#pragma unroll
      for (int i = 0; i < MB; ++i)
        fa[i] = *reinterpret_cast<const frag_t*>(stage + (a_base[i] ^ (ks << 5)));
#pragma unroll
      for (int j = 0; j < NB; ++j)
        fw[j] = *reinterpret_cast<const frag_t*>(stage + (w_base[j] ^ (ks << 5)));
#pragma unroll
      for (int i = 0; i < MB; ++i)
#pragma unroll
        for (int j = 0; j < NB; ++j)
          acc[i][j] = ROWS_IN_REGS ? mma32(T{}, fa[i], fw[j], acc[i][j])
                                   : mma32(T{}, fw[j], fa[i], acc[i][j]);
    }
    asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
  }

  if constexpr (ROWS_IN_REGS) {
#pragma unroll
    for (int i = 0; i < MB; ++i)
#pragma unroll
      for (int k = 0; k < 16; ++k) {
        const int r = rs.first + wm * (MB * 32) + i * 32 + 8 * (k >> 2) + 4 * g + (k & 3);
        if (r >= rs.last) continue;
        const long m = dst_row<MODE>(a, rs, r);
#pragma unroll
        for (int j = 0; j < NB; ++j) {
          const int n = n0 + wn * (NB * 32) + j * 32 + sigma(l32);
          if (n < a.N) store_col<TO>(a, m, n, finish<MODE>(a, n, acc[i][j][k]));
        }
      }
  } else {
#pragma unroll
    for (int i = 0; i < MB; ++i) {
      const int r = rs.first + wm * (MB * 32) + i * 32 + l32;
      if (r >= rs.last) continue;
      const long m = dst_row<MODE>(a, rs, r);
#pragma unroll
      for (int j = 0; j < (is_up(MODE) ? 1 : NB); ++j) {
        const int n = n0 + (is_up(MODE) ? wn * 32 : wn * (NB * 32) + j * 32) + 16 * g;
        float v[16];
#pragma unroll
        for (int k = 0; k < 16; ++k) {
          if constexpr (is_up(MODE)) v[k] = gated(a, acc[i][0][k], acc[i][1][k]);
          else v[k] = acc[i][j][k] * (MODE == kDense ? a.epi.scale : 1.f);
        }
        if (MODE == kDense && a.epi.bias) {
          if (n + 16 <= a.N) {
#pragma unroll
            for (int k = 0; k < 16; k += 4) {
              const f32x4 b = *reinterpret_cast<const f32x4*>(a.epi.bias + n + k);
#pragma unroll
              for (int e = 0; e < 4; ++e) v[k + e] += b[e];
            }
          } else {
#pragma unroll
            for (int k = 0; k < 16; ++k)
              if (n + k < a.N) v[k] += a.epi.bias[n + k];
          }
        }
        if (n + 16 <= min(a.N, a.n_split) && a.ldc % 8 == 0) {
          TO* p = reinterpret_cast<TO*>(a.C) + m * a.ldc + n;
          constexpr int V = 16 / sizeof(TO);
#pragma unroll
          for (int q = 0; q < 16 / V; ++q) {
            float t[V];
#pragma unroll
            for (int k = 0; k < V; ++k) t[k] = v[q * V + k];
            stv<V, TO>(p + q * V, t);
          }
        } else {
#pragma unroll
          for (int k = 0; k < 16; ++k)
            if (n + k < a.N) store_col<TO>(a, m, n + k, v[k]);
        }
      }
    }
  }
}

// ------------------------------------------------------------------------------------------------
// 16 * NS columns per workgroup (kDense; several strips share the activations), groups of 16 * MB
// rows; NW wavefronts split K.  HALVES (kGated): 8 columns, a fragment holds their gate rows and their
// up rows.  The weight fragment is the first operand: lane
// (c = lane % 16, q = lane / 16) holds column n0 + c's 16-byte chunk q of a 64-byte K slice.
template <typename T, typename TO, int MODE, int MB, int NS = 1, int NW = 4, bool HALVES = false>
__global__ void __launch_bounds__(64 * NW)
gemm_skinny_kernel(GemmArgs a) {
  static_assert(NS == 1 || MODE == kDense, "strips of one matrix");
  static_assert(!HALVES || MODE == kGated, "gate and up rows");
  constexpr int NB = is_up(MODE) && !HALVES ? 2 : NS;
  constexpr int V = FT<T>::kVec;
  // A turn takes U 64-byte slices of every row.  A wavefront loads whole lines, LR lanes to a row (a
  // fragment's lanes are 16 rows apart from each other in memory: loaded as such they would cost a
  // cache access each), and turns them into fragments in a part of LDS of its own.
  constexpr int U = (NB + MB) * NW <= 12 ? 4 : 2;
  constexpr int LR = 4 * U, RI = 64 / LR;        // lanes per row, rows per load
  constexpr int LW = 16 * NB / RI, LA = 16 * MB / RI;  // loads of weights, of activations
  constexpr int STR = U * 64 + 16;               // bytes from row to row in LDS
  constexpr int STAGE = 16 * (NB + MB) * STR;
  typedef float Red[NB][MB][16][17];
  constexpr int LDS = NW * STAGE > NW * (int)sizeof(Red) ? NW * STAGE : NW * (int)sizeof(Red);
  __shared__ __attribute__((aligned(16))) char smem[LDS];
  Red* red = reinterpret_cast<Red*>(smem);
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int c = lane & 15, q = lane >> 4;
  const int n0 = blockIdx.x * (HALVES ? 8 : 16 * NS);
  if (MODE == kDense && blockIdx.z == 1) {
    a.A = a.other.A;
    a.W = a.other.W;
    a.C = a.other.C;
    a.lda = a.other.lda;
    a.K = a.other.K;
    a.planes = a.other.planes;
    a.k_per_plane = a.other.k_per_plane;
  }
  if (MODE == kDense && (int)blockIdx.y >= a.planes) return;
  RowSet rs{0, 0, a.M};
  int k_lo = 0, k_hi = a.K;
  if (!is_dense(MODE)) {
    rs.expert = blockIdx.y;
    rs.last = a.count[rs.expert];
    if (rs.last == 0) return;
  } else {
    k_lo = blockIdx.y * a.k_per_plane;
    k_hi = min(a.K, k_lo + a.k_per_plane);
  }
  const T* W = reinterpret_cast<const T*>(a.W);
  if (!is_dense(MODE)) W += (long)rs.expert * NB * a.N * a.K;
  const int lr = lane / LR, lc = lane % LR;
  const T* wrow[LW];
#pragma unroll
  for (int i = 0; i < LW; ++i) {
    const int j = i * RI / 16, r = i * RI % 16 + lr;
    wrow[i] = W + lc * V +
              (HALVES ? (long)(min(n0 + (r & 7), a.N - 1) + (r >> 3) * a.N)
                      : is_up(MODE) ? (long)(min(n0 + r, a.N - 1) + j * a.N)
                                    : (long)min(n0 + j * 16 + r, a.N - 1)) * a.K;
  }
  const T* A = reinterpret_cast<const T*>(a.A);
  char* put = smem + wave * STAGE + lr * STR + lc * 16;
  const char* get = smem + wave * STAGE + c * STR + q * 16;
  const int first_end = rs.last;
  for (int first = 0; first < first_end; first += 16 * MB) {
    const T* arow[LA];
#pragma unroll
    for (int i = 0; i < LA; ++i) arow[i] = A + src_row<MODE>(a, rs, first + i * RI + lr) * a.lda + lc * V;
    f32x4 acc[NB][MB];
#pragma unroll
    for (int j = 0; j < NB; ++j)
#pragma unroll
      for (int i = 0; i < MB; ++i) acc[j][i] = (f32x4)0.f;
    frag_t lw[LW], la[LA];
    auto fetch = [&](int k) {
      const bool in = k + lc * V < k_hi;
#pragma unroll
      for (int i = 0; i < LW; ++i) lw[i] = in ? *reinterpret_cast<const frag_t*>(wrow[i] + k) : (frag_t)0u;
#pragma unroll
      for (int i = 0; i < LA; ++i) la[i] = in ? *reinterpret_cast<const frag_t*>(arow[i] + k) : (frag_t)0u;
    };
    constexpr int STEP = NW * U * 4 * V;
    int k = k_lo + wave * (U * 4 * V);
    if (k < k_hi) fetch(k);
    for (; k < k_hi; k += STEP) {
#pragma unroll
      for (int i = 0; i < LW; ++i) *reinterpret_cast<frag_t*>(put + i * RI * STR) = lw[i];
#pragma unroll
      for (int i = 0; i < LA; ++i) *reinterpret_cast<frag_t*>(put + (16 * NB + i * RI) * STR) = la[i];
      if (k + STEP < k_hi) fetch(k + STEP);
#pragma unroll
      for (int u = 0; u < U; ++u) {
        frag_t fw[NB], fa[MB];
#pragma unroll
        for (int j = 0; j < NB; ++j) fw[j] = *reinterpret_cast<const frag_t*>(get + j * 16 * STR + u * 64);
#pragma unroll
        for (int i = 0; i < MB; ++i)
          fa[i] = *reinterpret_cast<const frag_t*>(get + (NB + i) * 16 * STR + u * 64);
#pragma unroll
        for (int j = 0; j < NB; ++j)
#pragma unroll
          for (int i = 0; i < MB; ++i) acc[j][i] = mma16(T{}, fw[j], fa[i], acc[j][i]);
      }
    }
    __syncthreads();  // the sums take the place of the operands
#pragma unroll
    for (int j = 0; j < NB; ++j)
#pragma unroll
      for (int i = 0; i < MB; ++i)
#pragma unroll
        for (int v = 0; v < 4; ++v) red[wave][j][i][c][4 * q + v] = acc[j][i][v];
    __syncthreads();
    const int r = (tid >> 4) & 15;
#pragma unroll
    for (int i = tid >> 8; i < MB; i += NW / 4) {
      const int row = first + i * 16 + r;
      if (row >= rs.last) continue;
      float s[NB];
#pragma unroll
      for (int j = 0; j < NB; ++j) {
        s[j] = 0.f;
#pragma unroll
        for (int x = 0; x < NW; x += 4)
          s[j] += (red[x][j][i][r][tid & 15] + red[x + 1][j][i][r][tid & 15]) +
                  (red[x + 2][j][i][r][tid & 15] + red[x + 3][j][i][r][tid & 15]);
      }
      const long m = dst_row<MODE>(a, rs, row);
      if constexpr (HALVES) {
        const int n = n0 + (tid & 7);
        const float up = __shfl_xor(s[0], 8);  // a row's 16 lanes are all here
        if ((tid & 15) < 8 && n < a.N)
          reinterpret_cast<TO*>(a.C)[m * a.ldc + n] = from_f<TO>(gated(a, s[0], up));
      } else if constexpr (is_up(MODE)) {
        const int n = n0 + (tid & 15);
        if (n < a.N) reinterpret_cast<TO*>(a.C)[m * a.ldc + n] = from_f<TO>(gated(a, s[0], s[NB - 1]));
      } else {
#pragma unroll
        for (int j = 0; j < NB; ++j) {
          const int n = n0 + j * 16 + (tid & 15);
          if (n >= a.N) continue;
          if (MODE == kDense && a.planes > 1)
            reinterpret_cast<TO*>(a.C)[((long)blockIdx.y * a.M + m) * a.ldc + n] = from_f<TO>(s[j]);
          else
            store_col<TO>(a, m, n, finish<MODE>(a, n, s[j]));
        }
      }
    }
    __syncthreads();
  }
}

// ------------------------------------------------------------------------------------------------
// 64 x 64 tile, 4 wavefronts of 32 x 32, operands staged element by element with guards
template <typename T, typename TO, int MODE>
__global__ void __launch_bounds__(256)
gemm_generic_kernel(GemmArgs a, int tiles_n) {
  constexpr int NB = is_up(MODE) ? 2 : 1;
  constexpr int KS = 64 / sizeof(T);       // elements per K step
  constexpr int STR = 80 / sizeof(T);      // LDS row stride
  __shared__ __attribute__((aligned(16))) T As[64][STR], Ws[NB][64][STR];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int wm = wave >> 1, wn = wave & 1, c = lane & 15, q = lane >> 4;
  RowSet rs;
  const int tn = blockIdx.x % tiles_n, t = blockIdx.x / tiles_n;
  if (is_dense(MODE)) rs = RowSet{0, t * 64, min(a.M, t * 64 + 64)};
  else if (!expert_tile(a, t, 64, rs)) return;
  const int n0 = tn * 64;
  const T* A = reinterpret_cast<const T*>(a.A);
  const T* W = reinterpret_cast<const T*>(a.W);
  if (!is_dense(MODE)) W += (long)rs.expert * NB * a.N * a.K;
  f32x4 acc[NB][2][2];
#pragma unroll
  for (int j = 0; j < NB; ++j)
#pragma unroll
    for (int x = 0; x < 2; ++x)
#pragma unroll
      for (int y = 0; y < 2; ++y) acc[j][x][y] = (f32x4)0.f;
  const int row = tid >> 2;  // staged row, 4 threads each
  const T* ap = A + src_row<MODE>(a, rs, rs.first + row) * a.lda;
  const T* wp = W + (long)min(n0 + row, a.N - 1) * a.K;
  for (int k0 = 0; k0 < a.K; k0 += KS) {
    for (int e = tid & 3; e < KS; e += 4) {
      const bool in = k0 + e < a.K;
      As[row][e] = in ? ap[k0 + e] : from_f<T>(0.f);
#pragma unroll
      for (int j = 0; j < NB; ++j)
        Ws[j][row][e] = in ? wp[(long)j * a.N * a.K + k0 + e] : from_f<T>(0.f);
    }
    __syncthreads();
    frag_t fa[2];
#pragma unroll
    for (int x = 0; x < 2; ++x)
      fa[x] = *reinterpret_cast<const frag_t*>(&As[wm * 32 + x * 16 + c][q * FT<T>::kVec]);
#pragma unroll
    for (int j = 0; j < NB; ++j)
#pragma unroll
      for (int y = 0; y < 2; ++y) {
        const frag_t fw =
            *reinterpret_cast<const frag_t*>(&Ws[j][wn * 32 + y * 16 + c][q * FT<T>::kVec]);
#pragma unroll
        for (int x = 0; x < 2; ++x) acc[j][x][y] = mma16(T{}, fa[x], fw, acc[j][x][y]);
      }
    __syncthreads();
  }
#pragma unroll
  for (int x = 0; x < 2; ++x)
#pragma unroll
    for (int v = 0; v < 4; ++v) {
      const int r = rs.first + wm * 32 + x * 16 + 4 * q + v;
      if (r >= rs.last) continue;
      const long m = dst_row<MODE>(a, rs, r);
#pragma unroll
      for (int y = 0; y < 2; ++y) {
        const int n = n0 + wn * 32 + y * 16 + c;
        if (n >= a.N) continue;
        if constexpr (is_up(MODE))
          reinterpret_cast<TO*>(a.C)[m * a.ldc + n] =
              from_f<TO>(gated(a, acc[0][x][y][v], acc[NB - 1][x][y][v]));
        else
          store_col<TO>(a, m, n, finish<MODE>(a, n, acc[0][x][y][v]));
      }
    }
}

// ------------------------------------------------------------------------------------------------
template <typename T>
bool rows_aligned(const GemmArgs& a) {  // every row of A and W starts at 16 bytes
  return a.K % FT<T>::kVec == 0 && a.lda % FT<T>::kVec == 0 &&
         ((reinterpret_cast<uintptr_t>(a.A) | reinterpret_cast<uintptr_t>(a.W)) & 15u) == 0;
}
template <typename T>
bool tile_ok(const GemmArgs& a, int mode) {
  const long wrows = (long)(is_up(mode) ? 2 : 1) * a.N;
  const long arows = mode == kMoeDown ? (long)a.M * a.top : a.M;
  return rows_aligned<T>(a) && (long)a.K * sizeof(T) % kBK == 0 &&
         wrows * a.K * (long)sizeof(T) < (1L << 32) && arows * a.lda * (long)sizeof(T) < (1L << 32) &&
         ((reinterpret_cast<uintptr_t>(a.C) | reinterpret_cast<uintptr_t>(a.epi.bias)) & 15u) == 0;
}

template <typename T, typename TO, int MODE>
int launch_skinny(const GemmArgs& a, int rows, hipStream_t s) {
  const int strips = (a.N + 15) / 16;
  if constexpr (is_dense(MODE)) {
    const dim3 grid(strips, std::max(a.planes, a.other.planes), a.other.A ? 2 : 1);
    // a long K is split over eight wavefronts where there is at most a workgroup per compute unit
    const bool deep = a.planes == 1 && a.K * (int)sizeof(T) >= 2048;
    const bool wide = deep && strips <= cu_count();
    if constexpr (MODE == kDense) {
      if (a.planes == 1 && !a.other.A && rows > 16 && a.N >= 64 * cu_count()) {
        const dim3 half((a.N + 31) / 32, 1);
        if (rows <= 32) gemm_skinny_kernel<T, TO, MODE, 2, 2><<<half, 256, 0, s>>>(a);
        else gemm_skinny_kernel<T, TO, MODE, 4, 2><<<half, 256, 0, s>>>(a);
      } else if (rows <= 16) {
        if (wide) gemm_skinny_kernel<T, TO, MODE, 1, 1, 8><<<grid, 512, 0, s>>>(a);
        else gemm_skinny_kernel<T, TO, MODE, 1><<<grid, 256, 0, s>>>(a);
      } else if (rows <= 32) {
        if (wide) gemm_skinny_kernel<T, TO, MODE, 2, 1, 8><<<grid, 512, 0, s>>>(a);
        else gemm_skinny_kernel<T, TO, MODE, 2><<<grid, 256, 0, s>>>(a);
      } else {
        gemm_skinny_kernel<T, TO, MODE, 4><<<grid, 256, 0, s>>>(a);
      }
    } else {
      // strips of 8 columns fill the chip better, but read the activations twice as often
      const dim3 eights((a.N + 7) / 8);
      const bool halves = strips < (rows <= 16 ? 2 : 1) * cu_count();
#define GATED(MB)                                                                             \
  do {                                                                                        \
    if (halves && deep) gemm_skinny_kernel<T, TO, MODE, MB, 1, 8, true><<<eights, 512, 0, s>>>(a); \
    else if (halves) gemm_skinny_kernel<T, TO, MODE, MB, 1, 4, true><<<eights, 256, 0, s>>>(a);    \
    else if (wide) gemm_skinny_kernel<T, TO, MODE, MB, 1, 8><<<grid, 512, 0, s>>>(a);         \
    else gemm_skinny_kernel<T, TO, MODE, MB><<<grid, 256, 0, s>>>(a);                         \
  } while (0)
      if (rows <= 16) GATED(1);
      else if (rows <= 32) GATED(2);
      else gemm_skinny_kernel<T, TO, MODE, 4><<<grid, 256, 0, s>>>(a);
#undef GATED
    }
  } else {
    if (a.experts > 65535) return lsh_fail(LSH_ERR_UNSUPPORTED, "float gemm: too many experts");
    const dim3 grid(strips, a.experts);
    if (rows <= 16) gemm_skinny_kernel<T, TO, MODE, 1><<<grid, 256, 0, s>>>(a);
    else gemm_skinny_kernel<T, TO, MODE, 2><<<grid, 256, 0, s>>>(a);
  }
  return lsh_check_launch("gemm_skinny_kernel");
}

template <typename T, typename TO, int MODE>
int launch_any(const GemmArgs& a, hipStream_t s) {
  if (!a.A || !a.W || !a.C || a.M <= 0 || a.N <= 0 || a.K <= 0)
    return lsh_fail(LSH_ERR_INVALID, "float gemm: bad arguments");
  const long rows = is_dense(MODE) ? a.M : (long)a.M * a.top;
  // few rows per product: the weights are what is read
  if (rows_aligned<T>(a) && (is_dense(MODE) ? rows <= 64 : rows <= 24L * a.experts))
    return launch_skinny<T, TO, MODE>(a, is_dense(MODE) ? a.M : (int)rows / a.experts + 1, s);
  const auto tiles_m = [&](int tm) {  // upper bound: every expert may end in a part of a tile
    return is_dense(MODE) ? (rows + tm - 1) / tm : rows / tm + std::min((long)a.experts, rows);
  };
  if (tile_ok<T>(a, MODE)) {
    constexpr int kBigN = is_up(MODE) ? 64 : 128;
    const long big = tiles_m(128) * ((a.N + kBigN - 1) / kBigN);
    const bool small = is_dense(MODE) ? big < cu_count() : rows < 64L * a.experts;
    const int tm = small ? 64 : 128;
    const int tnn = is_up(MODE) ? 64 : small ? 64 : 128;
    const long gm = tiles_m(tm), gn = (a.N + tnn - 1) / tnn;
    if (gm * gn > 0x7fffffffL) return lsh_fail(LSH_ERR_UNSUPPORTED, "float gemm: too large");
    const unsigned grid = (unsigned)(gm * gn);
    if (small)
      gemm_tile_kernel<T, TO, MODE, 1, is_up(MODE) ? 2 : 1>
          <<<grid, 256, 0, s>>>(a, (int)gm, (int)gn);
    else
      gemm_tile_kernel<T, TO, MODE, 2, 2><<<grid, 256, 0, s>>>(a, (int)gm, (int)gn);
    return lsh_check_launch("gemm_tile_kernel");
  }
  const long gm = tiles_m(64), gn = (a.N + 63) / 64;
  if (gm * gn > 0x7fffffffL) return lsh_fail(LSH_ERR_UNSUPPORTED, "float gemm: too large");
  gemm_generic_kernel<T, TO, MODE><<<(unsigned)(gm * gn), 256, 0, s>>>(a, (int)gn);
  return lsh_check_launch("gemm_generic_kernel");
}

}  // namespace

template <typename T, typename TO>
int gemm_float(const T* A, long lda, const T* W, TO* C, long ldc, float* C2, long ld2, int n_split,
               int M, int N, int K, hipStream_t s, const GemmEpilogue& epilogue) {
  if (n_split < N && !C2) return lsh_fail(LSH_ERR_INVALID, "float gemm: no second output");
  GemmArgs a{};
  a.A = A; a.W = W; a.C = C; a.C2 = C2;
  a.lda = lda; a.ldc = ldc; a.ld2 = ld2; a.n_split = n_split;
  a.M = M; a.N = N; a.K = K;
  a.planes = 1; a.k_per_plane = K;
  a.epi = epilogue;
  return launch_any<T, TO, kDense>(a, s);
}

template <typename T>
int gemm_gated(const T* A, long lda, const T* W, T* C, long ldc, int M, int N, int K, int act,
               hipStream_t s) {
  if (act != kGateSilu && act != kGateRelu)
    return lsh_fail(LSH_ERR_INVALID, "gemm_gated: unknown activation");
  GemmArgs a{};
  a.A = A; a.W = W; a.C = C;
  a.lda = lda; a.ldc = ldc; a.n_split = N;
  a.M = M; a.N = N; a.K = K;
  a.planes = 1; a.k_per_plane = K;
  a.act = act;
  return launch_any<T, T, kGated>(a, s);
}

int gemm_float_preferred_planes(int M, int N, int K) {
  if (M > 64) return 1;
  const int strips = (N + 15) / 16;
  int p = 1;
  while (p < 8 && strips * p * 2 <= 2 * cu_count() && K / (2 * p) >= 256) p *= 2;
  return p;
}

namespace {

template <typename T>
GemmArgs planes_args(const FloatProduct<T>& p, int M, int N, int max_planes) {
  GemmArgs a{};
  a.A = p.A; a.W = p.W; a.C = p.C;
  a.lda = p.lda; a.ldc = N; a.n_split = N;
  a.M = M; a.N = N; a.K = p.K;
  a.planes = 1; a.k_per_plane = p.K;
  if (M <= 64 && max_planes > 1 && rows_aligned<T>(a)) {
    constexpr int step = 256 / sizeof(T);
    const int n = std::min(gemm_float_preferred_planes(M, N, p.K), max_planes);
    a.k_per_plane = ((p.K + n - 1) / n + step - 1) / step * step;
    a.planes = (p.K + a.k_per_plane - 1) / a.k_per_plane;
  }
  return a;
}

}  // namespace

template <typename T>
int gemm_float_planes(const T* A, long lda, const T* W, float* C, int M, int N, int K,
                      int max_planes, int* planes_used, hipStream_t s) {
  const GemmArgs a = planes_args(FloatProduct<T>{A, lda, W, C, K}, M, N, max_planes);
  *planes_used = a.planes;
  return launch_any<T, float, kDense>(a, s);
}

template <typename T>
int gemm_float_planes2(const FloatProduct<T>& p0, const FloatProduct<T>& p1, int M, int N,
                       int max_planes, int* planes0, int* planes1, hipStream_t s) {
  GemmArgs a = planes_args(p0, M, N, max_planes);
  const GemmArgs b = planes_args(p1, M, N, max_planes);
  *planes0 = a.planes;
  *planes1 = b.planes;
  if (!b.A || !b.W || !b.C || b.K <= 0 || M > 64 || !rows_aligned<T>(a) || !rows_aligned<T>(b)) {
    if (int rc = launch_any<T, float, kDense>(a, s)) return rc;
    return launch_any<T, float, kDense>(b, s);
  }
  a.other = {b.A, b.W, b.C, b.lda, b.K, b.planes, b.k_per_plane};
  return launch_any<T, float, kDense>(a, s);
}

template <typename T>
int moe_up(const T* h, const T* w, T* act, const int* count, const int* list, int tokens, int top,
           int experts, int width, int ff, hipStream_t s) {
  GemmArgs a{};
  a.A = h; a.W = w; a.C = act;
  a.lda = width; a.ldc = ff; a.n_split = ff;
  a.M = tokens; a.N = ff; a.K = width;
  a.count = count; a.list = list; a.list_stride = tokens; a.experts = experts; a.top = top;
  return launch_any<T, T, kMoeUp>(a, s);
}

template <typename T, typename TO>
int moe_down(const T* act, const T* w, TO* out, const int* count, const int* list, int tokens,
             int top, int experts, int width, int ff, hipStream_t s) {
  GemmArgs a{};
  a.A = act; a.W = w; a.C = out;
  a.lda = ff; a.ldc = width; a.n_split = width;
  a.M = tokens; a.N = width; a.K = ff;
  a.count = count; a.list = list; a.list_stride = tokens; a.experts = experts; a.top = top;
  return launch_any<T, TO, kMoeDown>(a, s);
}

#define INST_TT(T, TO)                                                                           \
  template int gemm_float<T, TO>(const T*, long, const T*, TO*, long, float*, long, int, int,    \
                                 int, int, hipStream_t, const GemmEpilogue&);                    \
  template int moe_down<T, TO>(const T*, const T*, TO*, const int*, const int*, int, int, int,   \
                               int, int, hipStream_t);
INST_TT(float, float)
INST_TT(bf16_t, bf16_t)
INST_TT(bf16_t, float)
#define INST_T(T)                                                                               \
  template int gemm_float_planes2<T>(const FloatProduct<T>&, const FloatProduct<T>&, int, int,  \
                                     int, int*, int*, hipStream_t);                             \
  template int gemm_gated<T>(const T*, long, const T*, T*, long, int, int, int, int,            \
                             hipStream_t);                                                      \
  template int gemm_float_planes<T>(const T*, long, const T*, float*, int, int, int, int, int*, \
                                    hipStream_t);                                               \
  template int moe_up<T>(const T*, const T*, T*, const int*, const int*, int, int, int, int, int, \
                         hipStream_t);
INST_T(float)
INST_T(bf16_t)

}  // namespace lsh
