// Routing of a mixture of experts: the largest logits of a token, the soft-max over them, and the
// list of rows every expert serves.  One wavefront per token, in float32.
#include "lm_launch.h"

namespace lsh {

namespace {

// The choices of one token by one wavefront: lane e % 64 holds logit e in z[e / 64] (-inf beyond the
// experts); lane j < top returns the j-th choice and its weight.
template <int EPL>
__device__ __forceinline__ void choose(const float (&z)[EPL], int experts, int top, int& my_e,
                                       float& my_w) {
  const int lane = threadIdx.x & 63;
  float my_z = -INFINITY;
  my_e = 0x7fffffff;
  unsigned taken = 0;  // this lane's logits already chosen
  for (int j = 0; j < top; ++j) {
    float m = -INFINITY;
#pragma unroll
    for (int i = 0; i < EPL; ++i)
      if (!(taken >> i & 1u)) m = fmaxf(m, z[i]);
    m = wave_max_dpp(m);
    int me = 0x7fffffff;  // the lowest index among the largest
#pragma unroll
    for (int i = EPL - 1; i >= 0; --i) {
      const unsigned long long hit =
          __ballot(!(taken >> i & 1u) && i * 64 + lane < experts && z[i] == m);
      if (hit) me = i * 64 + __ffsll(hit) - 1;
    }
    if ((me & 63) == lane) taken |= 1u << ((me >> 6) & 31);
    if (lane == j) {
      my_z = m;
      my_e = me;
    }
  }
  const float ex = lane < top ? expf(my_z - __shfl(my_z, 0)) : 0.f;
  my_w = ex / wave_sum(ex);
}

// A workgroup takes NW * TPW tokens and counts its choices in LDS first, so that an expert's counter
// sees one addition per workgroup.  EPL logits per lane: experts <= 64 * EPL.
template <int EPL, int TPW, int NW>
__global__ void __launch_bounds__(64 * NW)
moe_route_kernel(const float* __restrict__ logits, const float* __restrict__ bias,
                 float* __restrict__ weight, int* __restrict__ count, int* __restrict__ list,
                 int tokens, int experts, int top) {
  __shared__ int cnt[64 * EPL], base[64 * EPL];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  for (int e = threadIdx.x; e < experts; e += 64 * NW) cnt[e] = 0;
  __syncthreads();
  const int t0 = (blockIdx.x * NW + wave) * TPW;
  float z[TPW][EPL];
#pragma unroll
  for (int u = 0; u < TPW; ++u)
#pragma unroll
    for (int i = 0; i < EPL; ++i) {
      const int e = i * 64 + lane;
      z[u][i] = e < experts ? logits[(long)min(t0 + u, tokens - 1) * experts + e] +
                                  (bias ? bias[e] : 0.f)
                            : -INFINITY;
    }
  int my_e[TPW], rank[TPW];
#pragma unroll
  for (int u = 0; u < TPW; ++u) {
    const int t = t0 + u;
    my_e[u] = -1;
    rank[u] = 0;
    if (t < tokens) {
      float w;
      int e;
      choose<EPL>(z[u], experts, top, e, w);
      if (lane < top) {
        weight[(long)t * top + lane] = w;
        if (e < experts) {  // always, for finite logits
          my_e[u] = e;
          rank[u] = atomicAdd(&cnt[e], 1);
        }
      }
    }
  }
  __syncthreads();
  for (int e = threadIdx.x; e < experts; e += 64 * NW)
    if (cnt[e] > 0) base[e] = atomicAdd(&count[e], cnt[e]);
  __syncthreads();
#pragma unroll
  for (int u = 0; u < TPW; ++u)
    if (my_e[u] >= 0) {
      const int t = t0 + u;
      list[(long)my_e[u] * tokens + base[my_e[u]] + rank[u]] = t * top + lane;
    }
}

// The router product and the choice of one token by one workgroup (few tokens).  The dot products are
// spread over the wavefronts, their lanes along the width.
template <typename T, int EPL>
__global__ void __launch_bounds__(256)
moe_router_kernel(const T* __restrict__ h, const T* __restrict__ w, const float* __restrict__ bias,
                  float* __restrict__ weight, int* __restrict__ count, int* __restrict__ list,
                  int tokens, int width, int experts, int top) {
  constexpr int V = FT<T>::kVec;
  __shared__ float z_s[64 * EPL];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, t = blockIdx.x;
  const T* hr = h + (long)t * width;
  const bool vec = width % V == 0;
  for (int e0 = wave * 4; e0 < experts; e0 += 16) {  // four rows at once: their loads overlap
    float d[4] = {0.f, 0.f, 0.f, 0.f};
    const T* wr[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) wr[u] = w + (long)min(e0 + u, experts - 1) * width;
    if (vec) {
      for (int k = lane * V; k < width; k += 64 * V) {
        float x[V], y[V];
        ldv<V, T>(hr + k, x);
#pragma unroll
        for (int u = 0; u < 4; ++u) {
          ldv<V, T>(wr[u] + k, y);
#pragma unroll
          for (int i = 0; i < V; ++i) d[u] = fmaf(x[i], y[i], d[u]);
        }
      }
    } else {
      for (int k = lane; k < width; k += 64)
#pragma unroll
        for (int u = 0; u < 4; ++u) d[u] = fmaf(to_f(hr[k]), to_f(wr[u][k]), d[u]);
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const float s = wave_sum_dpp(d[u]);
      if (lane == 0 && e0 + u < experts) z_s[e0 + u] = s + (bias ? bias[e0 + u] : 0.f);
    }
  }
  __syncthreads();
  if (wave != 0) return;
  float z[EPL], wt;
#pragma unroll
  for (int i = 0; i < EPL; ++i) z[i] = i * 64 + lane < experts ? z_s[i * 64 + lane] : -INFINITY;
  int e;
  choose<EPL>(z, experts, top, e, wt);
  if (lane < top) {
    weight[(long)t * top + lane] = wt;
    if (e < experts) list[(long)e * tokens + atomicAdd(&count[e], 1)] = t * top + lane;
  }
}

int check(int tokens, int experts, int top) {
  if (tokens <= 0 || experts <= 0 || top <= 0)
    return lsh_fail(LSH_ERR_INVALID, "moe routing: bad arguments");
  if (top > 64 || top > experts || experts > 1024)
    return lsh_fail(LSH_ERR_UNSUPPORTED, "moe routing: at most 64 choices of at most 1024 experts");
  return LSH_OK;
}

}  // namespace

int moe_route(const float* logits, const float* bias, float* weight, int* count, int* list,
              int tokens, int experts, int top, hipStream_t s) {
  if (int rc = check(tokens, experts, top)) return rc;
  if (!logits || !weight || !count || !list)
    return lsh_fail(LSH_ERR_INVALID, "moe_route: bad arguments");
#define ROUTE(EPL, TPW, NW)                                                                      \
  moe_route_kernel<EPL, TPW, NW><<<(tokens + NW * TPW - 1) / (NW * TPW), 64 * NW, 0, s>>>(       \
      logits, bias, weight, count, list, tokens, experts, top)
  const bool many = tokens >= 512;
  if (experts <= 64) {
    if (many) ROUTE(1, 8, 16);
    else ROUTE(1, 1, 4);
  } else if (experts <= 256) {
    if (many) ROUTE(4, 4, 16);
    else ROUTE(4, 1, 4);
  } else {
    ROUTE(16, 1, 4);
  }
#undef ROUTE
  return lsh_check_launch("moe_route_kernel");
}

template <typename T>
int moe_router(const T* h, const T* w, const float* bias, float* weight, int* count, int* list,
               int tokens, int width, int experts, int top, hipStream_t s) {
  if (int rc = check(tokens, experts, top)) return rc;
  if (!h || !w || !weight || !count || !list || width <= 0)
    return lsh_fail(LSH_ERR_INVALID, "moe_router: bad arguments");
#define ROUTER(EPL) \
  moe_router_kernel<T, EPL><<<tokens, 256, 0, s>>>(h, w, bias, weight, count, list, tokens, width, experts, top)
  if (experts <= 64) ROUTER(1);
  else if (experts <= 256) ROUTER(4);
  else ROUTER(16);
#undef ROUTER
  return lsh_check_launch("moe_router_kernel");
}
template int moe_router<float>(const float*, const float*, const float*, float*, int*, int*, int,
                               int, int, int, hipStream_t);
template int moe_router<bf16_t>(const bf16_t*, const bf16_t*, const float*, float*, int*, int*, int,
                                int, int, int, hipStream_t);

}  // namespace lsh
