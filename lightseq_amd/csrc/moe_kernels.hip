// Routing of a mixture of experts: the largest logits of a token, the soft-max over them, and the
// list of rows every expert serves.  One wavefront per token, in float32.
#include "lm_launch.h"

namespace lsh {

namespace {

// EPL logits per lane: experts <= 64 * EPL
template <int EPL>
__global__ void __launch_bounds__(256)
moe_route_kernel(const float* __restrict__ logits, const float* __restrict__ bias,
                 float* __restrict__ weight, int* __restrict__ count, int* __restrict__ list,
                 int tokens, int experts, int top) {
  const int lane = threadIdx.x & 63;
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (t >= tokens) return;
  float z[EPL];
#pragma unroll
  for (int i = 0; i < EPL; ++i) {
    const int e = i * 64 + lane;
    z[i] = e < experts ? logits[(long)t * experts + e] + (bias ? bias[e] : 0.f) : -INFINITY;
  }
  // lane j keeps the j-th choice
  float my_z = -INFINITY;
  int my_e = 0;
  unsigned taken = 0;  // this lane's logits already chosen
  for (int j = 0; j < top; ++j) {
    float m = -INFINITY;
    int me = 0x7fffffff;
#pragma unroll
    for (int i = 0; i < EPL; ++i)
      if (!(taken >> i & 1u) && i * 64 + lane < experts && (z[i] > m || me == 0x7fffffff)) {
        m = z[i];
        me = i * 64 + lane;
      }
#pragma unroll
    for (int d = 32; d > 0; d >>= 1) {
      const float om = __shfl_xor(m, d);
      const int oe = __shfl_xor(me, d);
      if (om > m || (om == m && oe < me)) {
        m = om;
        me = oe;
      }
    }
    if ((me & 63) == lane) taken |= 1u << (me >> 6);
    if (lane == j) {
      my_z = m;
      my_e = me;
    }
  }
  const float mx = __shfl(my_z, 0);
  const float ex = lane < top ? expf(my_z - mx) : 0.f;
  const float sum = wave_sum(ex);
  if (lane < top) {
    weight[(long)t * top + lane] = ex / sum;
    if (my_e < experts) {
      const int at = atomicAdd(&count[my_e], 1);
      list[(long)my_e * tokens + at] = t * top + lane;
    }
  }
}

}  // namespace

int moe_route(const float* logits, const float* bias, float* weight, int* count, int* list,
              int tokens, int experts, int top, hipStream_t s) {
  if (!logits || !weight || !count || !list || tokens <= 0 || experts <= 0 || top <= 0)
    return lsh_fail(LSH_ERR_INVALID, "moe_route: bad arguments");
  if (top > 64 || top > experts || experts > 1024)
    return lsh_fail(LSH_ERR_UNSUPPORTED, "moe_route: at most 64 choices of at most 1024 experts");
  const int grid = (tokens + 3) / 4;
  if (experts <= 64)
    moe_route_kernel<1><<<grid, 256, 0, s>>>(logits, bias, weight, count, list, tokens, experts, top);
  else if (experts <= 256)
    moe_route_kernel<4><<<grid, 256, 0, s>>>(logits, bias, weight, count, list, tokens, experts, top);
  else
    moe_route_kernel<16><<<grid, 256, 0, s>>>(logits, bias, weight, count, list, tokens, experts, top);
  return lsh_check_launch("moe_route_kernel");
}

}  // namespace lsh
