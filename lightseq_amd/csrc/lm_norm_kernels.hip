// The residual stream of a floating-point decoder and its norms, in float32: one workgroup
// per row, the row in registers.  One launch adds a sublayer's output to the residual (after that
// sublayer's own norm, from partial sums or weighted expert outputs as they lie in memory; or that of
// two sublayers side by side) and applies the norm ahead of the next sublayer; another starts the
// stream from the embedding table.
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
  InjectSpec inject;
};

// V elements per access, NI accesses per thread: width <= 256 * V * NI
template <typename T, typename TY, int V, int NI>
__global__ void __launch_bounds__(256)
lm_norm_kernel(NormArgs a) {
  __shared__ float red[6][16];
  const int tid = threadIdx.x, W = a.width;
  const long r = blockIdx.x;
  if (r == 0 && a.n_zero > 0)
    for (int i = tid; i < a.n_zero; i += 256) a.zero_count[i] = 0;
  float* xr = a.x + (a.rows ? (long)a.rows[r] : r) * W;
  float x[NI][V];
  const auto embed_row = [&](const int* ids) {
    return ids ? reinterpret_cast<const T*>(a.embed) + (long)min(max(ids[r], 0), a.vocab - 1) * W
               : nullptr;
  };
  const T* er = embed_row(a.ids);
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
  // mean and reciprocal deviation of a row held as v (zeros beyond the width); 0 and the reciprocal
  // root mean square
  auto stats = [&](const float (&v)[NI][V], NormKind kind, float& mean, float& rstd, int which) {
    float s = 0.f;
    if (kind == kRmsNorm) {
#pragma unroll
      for (int i = 0; i < NI; ++i)
#pragma unroll
        for (int k = 0; k < V; ++k) s += v[i][k] * v[i][k];
      mean = 0.f;
      rstd = 1.0f / sqrtf(block_sum_dpp(s, red[which]) * inv_w + a.eps);
      return;
    }
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
  // the sum of a summand's pieces, PU of them requested at a time
  constexpr int PU = NI <= 2 ? 4 : NI <= 4 ? 2 : 1;
  auto gather = [&](const AddPart& part, float (&y)[NI][V]) {
#pragma unroll
    for (int i = 0; i < NI; ++i)
#pragma unroll
      for (int k = 0; k < V; ++k) y[i][k] = 0.f;
    const TY* yr = reinterpret_cast<const TY*>(part.y) + r * part.row_stride;
    if (part.parts == 1 && !part.weight) {
#pragma unroll
      for (int i = 0; i < NI; ++i) {
        const int c = (i * 256 + tid) * V;
        if (c < W) ldv<V, TY>(yr + c, y[i]);
      }
      return;
    }
    for (int p0 = 0; p0 < part.parts; p0 += PU) {
      float t[PU][NI][V], wt[PU];
#pragma unroll
      for (int u = 0; u < PU; ++u) {
        const bool there = p0 + u < part.parts;
        wt[u] = there && part.weight ? part.weight[r * part.parts + p0 + u] : 1.f;
#pragma unroll
        for (int i = 0; i < NI; ++i) {
          const int c = (i * 256 + tid) * V;
#pragma unroll
          for (int k = 0; k < V; ++k) t[u][i][k] = 0.f;
          if (there && c < W) ldv<V, TY>(yr + (p0 + u) * part.part_stride + c, t[u][i]);
        }
      }
#pragma unroll
      for (int u = 0; u < PU; ++u)
#pragma unroll
        for (int i = 0; i < NI; ++i)
#pragma unroll
          for (int k = 0; k < V; ++k) y[i][k] += wt[u] * t[u][i][k];
    }
  };
  auto add = [&](const AddPart& part, const float (&y)[NI][V], int which) {
    float mean = 0.f, rstd = 1.f;
    if (part.post_w) stats(y, a.add.post_kind, mean, rstd, which);
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int c = (i * 256 + tid) * V;
      if (c < W) {
        if (part.post_w) {
          float w[V], b[V];
          ldv<V, float>(part.post_w + c, w);
#pragma unroll
          for (int k = 0; k < V; ++k) b[k] = 0.f;
          if (part.post_b) ldv<V, float>(part.post_b + c, b);
#pragma unroll
          for (int k = 0; k < V; ++k) x[i][k] += a.add.scale * ((y[i][k] - mean) * rstd * w[k] + b[k]);
        } else {
#pragma unroll
          for (int k = 0; k < V; ++k) x[i][k] += a.add.scale * y[i][k];
        }
      }
    }
  };
  if (a.add.parts > 0) {
    float y[NI][V];
    gather(a.add, y);
    if (a.add.second.parts > 0) {
      float z[NI][V];
      gather(a.add.second, z);
      add(a.add, y, 0);
      add(a.add.second, z, 2);
    } else {
      add(a.add, y, 0);
    }
  }
  if (a.inject.any()) {
    const T* ir = embed_row(a.inject.ids);
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int c = (i * 256 + tid) * V;
      if (c < W) {
        float t[V];
        if (ir) {
          ldv<V, T>(ir + c, t);
#pragma unroll
          for (int k = 0; k < V; ++k) x[i][k] += t[k];
        }
        if (a.inject.vec) {
          ldv<V, float>(a.inject.vec + c, t);
#pragma unroll
          for (int k = 0; k < V; ++k) x[i][k] += t[k];
        }
      }
    }
  }
  if (a.add.parts > 0 || a.ids || a.inject.any()) {
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int c = (i * 256 + tid) * V;
      if (c < W) stv<V, float>(xr + c, x[i]);
    }
  }
  if (!a.norm.w) return;
  float mean, rstd;
  stats(x, a.norm.kind, mean, rstd, 4);
  T* hr = reinterpret_cast<T*>(a.h) + r * W;
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int c = (i * 256 + tid) * V;
    if (c < W) {
      float w[V], b[V], o[V];
      ldv<V, float>(a.norm.w + c, w);
#pragma unroll
      for (int k = 0; k < V; ++k) b[k] = 0.f;
      if (a.norm.b) ldv<V, float>(a.norm.b + c, b);
#pragma unroll
      for (int k = 0; k < V; ++k) o[k] = (x[i][k] - mean) * rstd * w[k] + b[k];
      stv<V, T>(hr + c, o);
    }
  }
}

template <typename T, typename TY>
int launch_norm(const NormArgs& a, int rows, hipStream_t s) {
  const bool vec = a.width % 4 == 0 && a.add.part_stride % 4 == 0 && a.add.row_stride % 4 == 0 &&
                   a.add.second.part_stride % 4 == 0 && a.add.second.row_stride % 4 == 0;
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
            int n_zero, hipStream_t s, const InjectSpec& inject) {
  const bool adds = add.parts > 0 || add.second.parts > 0 || inject.any();
  if (!x || rows_n <= 0 || width <= 0 || ((ids || inject.ids) && (!embed || vocab <= 0)) ||
      (add.parts > 0 && !add.y) || (add.second.parts > 0 && (add.parts <= 0 || !add.second.y)) ||
      (norm.w && !h) || (rows && (adds || ids)) ||
      (norm.w && norm.kind == kLayerNorm && !norm.b) ||
      (add.post_w && add.post_kind == kLayerNorm && !add.post_b) ||
      (add.second.post_w && add.post_kind == kLayerNorm && !add.second.post_b))
    return lsh_fail(LSH_ERR_INVALID, "lm_norm: bad arguments");
  const NormArgs a{x, add, norm, h, width, eps, ids, embed, vocab, rows, zero_count,
                   zero_count ? n_zero : 0, inject};
  return add.y_is_float ? launch_norm<T, float>(a, rows_n, s) : launch_norm<T, T>(a, rows_n, s);
}
template int lm_norm<float>(float*, const AddSpec&, const NormSpec&, float*, int, int, float,
                            const int*, const float*, int, const int*, int*, int, hipStream_t,
                            const InjectSpec&);
template int lm_norm<bf16_t>(float*, const AddSpec&, const NormSpec&, bf16_t*, int, int, float,
                             const int*, const bf16_t*, int, const int*, int*, int, hipStream_t,
                             const InjectSpec&);

}  // namespace lsh
