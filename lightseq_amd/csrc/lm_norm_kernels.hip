// The residual stream of a floating-point decoder and its layer norms, in float32: one workgroup
// per row, the row in registers.  One launch adds a sublayer's output to the residual (after that
// sublayer's own norm, from partial sums or weighted expert outputs as they lie in memory) and
// applies the norm ahead of the next sublayer; another starts the stream from the embedding table.
#include "lm_launch.h"

namespace lsh {

namespace {

struct NormArgs {
  float* x;
  AddSpec add;
  NormSpec norm;
  void* h;
  int width;
  float eps;
  const int* ids;
  const void* embed;
  int vocab;
  const int* rows;
  int* zero_count;
  int n_zero;
};

// V elements per access, NI accesses per thread: width <= 256 * V * NI
template <typename T, typename TY, int V, int NI>
__global__ void __launch_bounds__(256)
lm_norm_kernel(NormArgs a) {
  __shared__ float red[4][16];
  const int tid = threadIdx.x, W = a.width;
  const long r = blockIdx.x;
  if (r == 0 && a.n_zero > 0)
    for (int i = tid; i < a.n_zero; i += 256) a.zero_count[i] = 0;
  float* xr = a.x + (a.rows ? (long)a.rows[r] : r) * W;
  float x[NI][V];
  const T* er = nullptr;
  if (a.ids) {
    const int id = a.ids[r];
    er = reinterpret_cast<const T*>(a.embed) + (long)min(max(id, 0), a.vocab - 1) * W;
  }
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int c = (i * 256 + tid) * V;
#pragma unroll
    for (int k = 0; k < V; ++k) x[i][k] = 0.f;
    if (c < W) {
      if (er) ldv<V, T>(er + c, x[i]);
      else ldv<V, float>(xr + c, x[i]);
    }
  }
  const float inv_w = 1.f / (float)W;
  // mean and reciprocal deviation of a row held as v
  auto stats = [&](const float (&v)[NI][V], float& mean, float& rstd, int which) {
    float s = 0.f;
#pragma unroll
    for (int i = 0; i < NI; ++i)
#pragma unroll
      for (int k = 0; k < V; ++k) s += v[i][k];
    mean = block_sum_dpp(s, red[which]) * inv_w;
    s = 0.f;
#pragma unroll
    for (int i = 0; i < NI; ++i)
      if ((i * 256 + tid) * V < W) {
#pragma unroll
        for (int k = 0; k < V; ++k) {
          const float d = v[i][k] - mean;
          s += d * d;
        }
      }
    rstd = 1.0f / sqrtf(block_sum_dpp(s, red[which + 1]) * inv_w + a.eps);
  };
  if (a.add.parts > 0) {
    float y[NI][V];
#pragma unroll
    for (int i = 0; i < NI; ++i)
#pragma unroll
      for (int k = 0; k < V; ++k) y[i][k] = 0.f;
    const TY* yr = reinterpret_cast<const TY*>(a.add.y) + r * a.add.row_stride;
    for (int p = 0; p < a.add.parts; ++p) {
      const float wt = a.add.weight ? a.add.weight[r * a.add.parts + p] : 1.f;
#pragma unroll
      for (int i = 0; i < NI; ++i) {
        const int c = (i * 256 + tid) * V;
        if (c < W) {
          float t[V];
          ldv<V, TY>(yr + p * a.add.part_stride + c, t);
#pragma unroll
          for (int k = 0; k < V; ++k) y[i][k] += wt * t[k];
        }
      }
    }
    float mean = 0.f, rstd = 1.f;
    if (a.add.post_w) stats(y, mean, rstd, 0);
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int c = (i * 256 + tid) * V;
      if (c < W) {
        if (a.add.post_w) {
          float w[V], b[V];
          ldv<V, float>(a.add.post_w + c, w);
          ldv<V, float>(a.add.post_b + c, b);
#pragma unroll
          for (int k = 0; k < V; ++k) x[i][k] += (y[i][k] - mean) * rstd * w[k] + b[k];
        } else {
#pragma unroll
          for (int k = 0; k < V; ++k) x[i][k] += y[i][k];
        }
      }
    }
  }
  if (a.add.parts > 0 || a.ids) {
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int c = (i * 256 + tid) * V;
      if (c < W) stv<V, float>(xr + c, x[i]);
    }
  }
  if (!a.norm.w) return;
  float mean, rstd;
  stats(x, mean, rstd, 2);
  T* hr = reinterpret_cast<T*>(a.h) + r * W;
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int c = (i * 256 + tid) * V;
    if (c < W) {
      float w[V], b[V], o[V];
      ldv<V, float>(a.norm.w + c, w);
      ldv<V, float>(a.norm.b + c, b);
#pragma unroll
      for (int k = 0; k < V; ++k) o[k] = (x[i][k] - mean) * rstd * w[k] + b[k];
      stv<V, T>(hr + c, o);
    }
  }
}

template <typename T, typename TY>
int launch_norm(const NormArgs& a, int rows, hipStream_t s) {
  const bool vec = a.width % 4 == 0 && a.add.part_stride % 4 == 0 && a.add.row_stride % 4 == 0;
  const int per = 256 * (vec ? 4 : 1);
  const int ni = (a.width + per - 1) / per;
  if (vec) {
    if (ni <= 1) lm_norm_kernel<T, TY, 4, 1><<<rows, 256, 0, s>>>(a);
    else if (ni <= 2) lm_norm_kernel<T, TY, 4, 2><<<rows, 256, 0, s>>>(a);
    else if (ni <= 4) lm_norm_kernel<T, TY, 4, 4><<<rows, 256, 0, s>>>(a);
    else if (ni <= 8) lm_norm_kernel<T, TY, 4, 8><<<rows, 256, 0, s>>>(a);
    else return lsh_fail(LSH_ERR_UNSUPPORTED, "lm_norm: width above 8192");
  } else {
    if (ni <= 8) lm_norm_kernel<T, TY, 1, 8><<<rows, 256, 0, s>>>(a);
    else if (ni <= 16) lm_norm_kernel<T, TY, 1, 16><<<rows, 256, 0, s>>>(a);
    else return lsh_fail(LSH_ERR_UNSUPPORTED, "lm_norm: width above 4096 and not a multiple of 4");
  }
  return lsh_check_launch("lm_norm_kernel");
}

}  // namespace

template <typename T>
int lm_norm(float* x, const AddSpec& add, const NormSpec& norm, T* h, int rows_n, int width,
            float eps, const int* ids, const T* embed, int vocab, const int* rows, int* zero_count,
            int n_zero, hipStream_t s) {
  if (!x || rows_n <= 0 || width <= 0 || (ids && !embed) || (add.parts > 0 && !add.y) ||
      (norm.w && (!norm.b || !h)) || (add.post_w && !add.post_b) || (rows && (add.parts > 0 || ids)))
    return lsh_fail(LSH_ERR_INVALID, "lm_norm: bad arguments");
  const NormArgs a{x, add, norm, h, width, eps, ids, embed, vocab, rows, zero_count,
                   zero_count ? n_zero : 0};
  return add.y_is_float ? launch_norm<T, float>(a, rows_n, s) : launch_norm<T, T>(a, rows_n, s);
}
template int lm_norm<float>(float*, const AddSpec&, const NormSpec&, float*, int, int, float,
                            const int*, const float*, int, const int*, int*, int, hipStream_t);
template int lm_norm<bf16_t>(float*, const AddSpec&, const NormSpec&, bf16_t*, int, int, float,
                             const int*, const bf16_t*, int, const int*, int*, int, hipStream_t);

}  // namespace lsh
