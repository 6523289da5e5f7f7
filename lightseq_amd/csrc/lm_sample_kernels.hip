// Choice of the next token from float32 logits: greedy, top-k or top-p, one workgroup per row, with
// the library's Philox streams (sample_common.h).  Candidates are taken in descending order of
// logit; of equal logits the lower id comes first.
#include "lm_launch.h"
#include "sample_common.h"

namespace lsh {

namespace {

struct Best {
  float z;
  int id;
};
__device__ __forceinline__ bool before(float z, int id, float z2, int id2) {
  return z > z2 || (z == z2 && id < id2);
}
__device__ __forceinline__ Best wave_best(Best b) {
#pragma unroll
  for (int d = 32; d > 0; d >>= 1) {
    const float z = __shfl_xor(b.z, d);
    const int id = __shfl_xor(b.id, d);
    if (before(z, id, b.z, b.id)) b = Best{z, id};
  }
  return b;
}

struct SampleLds {
  float red[16];
  float bz[16];
  int bid[16];
  float pre[16];
  float x;
  int tok;
};

// the first candidate in that order which comes after (z, id)
__device__ Best next_best(const float* lr, int vocab, float z, int id, SampleLds& sh) {
  Best b{-INFINITY, 0x7fffffff};
  if (vocab % 4 == 0) {  // rows start at 16 bytes
    const int quads = vocab / 4;
    for (int v0 = threadIdx.x; v0 < quads; v0 += 4 * blockDim.x) {
      float4 t[4];
#pragma unroll
      for (int u = 0; u < 4; ++u)
        t[u] = reinterpret_cast<const float4*>(lr)[min(v0 + u * (int)blockDim.x, quads - 1)];
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int v = min(v0 + u * (int)blockDim.x, quads - 1) * 4;
        const float x[4] = {t[u].x, t[u].y, t[u].z, t[u].w};
#pragma unroll
        for (int k = 0; k < 4; ++k)
          if (before(z, id, x[k], v + k) && before(x[k], v + k, b.z, b.id)) b = Best{x[k], v + k};
      }
    }
  } else {
    for (int v = threadIdx.x; v < vocab; v += blockDim.x) {
      const float x = lr[v];
      if (before(z, id, x, v) && before(x, v, b.z, b.id)) b = Best{x, v};
    }
  }
  b = wave_best(b);
  const int wid = threadIdx.x >> 6, nw = blockDim.x >> 6;
  __syncthreads();
  if ((threadIdx.x & 63) == 0) {
    sh.bz[wid] = b.z;
    sh.bid[wid] = b.id;
  }
  __syncthreads();
  for (int i = 0; i < nw; ++i)
    if (before(sh.bz[i], sh.bid[i], b.z, b.id)) b = Best{sh.bz[i], sh.bid[i]};
  return b;
}

__global__ void __launch_bounds__(1024)
lm_sample_kernel(const float* __restrict__ logits, int vocab, int topk, float topp, int eos_id,
                 SampleState* __restrict__ rng, int* __restrict__ ids, int max_step,
                 int* __restrict__ last_ids, int* __restrict__ row_len, int* __restrict__ row_pos,
                 int* __restrict__ unfinished) {
  __shared__ SampleLds sh;
  const int row = blockIdx.x, tid = threadIdx.x;
  const int len = row_len[row];
  // an ended row stays as it is: its text does not grow and its position does not move
  if (len < 0) return;
  const float* lr = logits + (long)row * vocab;
  Best top = next_best(lr, vocab, INFINITY, -1, sh);
  int tok = top.id;
  if (topk != 1) {
    Best lim = top;  // the last candidate
    if (topk > 1) {
      for (int i = 1; i < topk && i < vocab; ++i) lim = next_best(lr, vocab, lim.z, lim.id, sh);
    } else {
      // the smallest logit whose candidates, from the largest down, hold no more than topp of the
      // probability before it is counted in: by bisection on the logit
      float all = 0.f;
      for (int v = tid; v < vocab; v += blockDim.x) all += expf(lr[v] - top.z);
      all = block_sum(all, sh.red);
      float lo = top.z - 64.f, hi = top.z;  // mass of {z > hi} < topp <= mass of {z > lo}
      for (int it = 0; it < 40; ++it) {
        const float mid = 0.5f * (lo + hi);
        float m = 0.f;
        for (int v = tid; v < vocab; v += blockDim.x)
          if (lr[v] > mid) m += expf(lr[v] - top.z);
        m = block_sum(m, sh.red);
        if (m < topp * all) hi = mid;
        else lo = mid;
      }
      lim = Best{lo, -1};  // candidates: z > lo
    }
    // every thread owns a contiguous run of ids, so prefixes are in id order
    const int per = (vocab + (int)blockDim.x - 1) / (int)blockDim.x;
    const int v0 = min(tid * per, vocab), v1 = min(v0 + per, vocab);
    float mine = 0.f;
    for (int v = v0; v < v1; ++v)
      if (!before(lim.z, lim.id, lr[v], v)) mine += expf(lr[v] - top.z);
    float pre = mine;
    const int lane = tid & 63, wid = tid >> 6;
#pragma unroll
    for (int d = 1; d < 64; d <<= 1) {
      const float up = __shfl_up(pre, d);
      if (lane >= d) pre += up;
    }
    if (tid == 0) {
      sh.x = sample_draw_uniform(&rng[row]);
      sh.tok = top.id;  // kept if rounding leaves no prefix at the drawn number
    }
    if (lane == 63) sh.pre[wid] = pre;
    __syncthreads();
    float total = 0.f;
    for (int w = 0; w < (int)(blockDim.x >> 6); ++w) {
      if (w < wid) pre += sh.pre[w];
      total += sh.pre[w];
    }
    const float x = sh.x * total;
    if (mine > 0.f && x > pre - mine && x <= pre) {
      float c = pre - mine;
      int last = -1;
      for (int v = v0; v < v1; ++v)
        if (!before(lim.z, lim.id, lr[v], v)) {
          last = v;
          c += expf(lr[v] - top.z);
          if (c >= x) break;
        }
      sh.tok = last;
    }
    __syncthreads();
    tok = sh.tok;
  }
  if (tid == 0) {
    ids[(long)row * max_step + len] = tok;
    last_ids[row] = tok;
    if (tok == eos_id) {
      row_len[row] = -(len + 1);  // ended with len + 1 ids
    } else {
      row_len[row] = len + 1;
      *unfinished = 1;
    }
    row_pos[row] = len;  // where the chosen token goes when it is fed back
  }
}

}  // namespace

int lm_sample(const float* logits, int rows, int vocab, int topk, float topp, int eos_id,
              void* rng_state, int* ids, int max_step, int* last_ids, int* row_len, int* row_pos,
              int* unfinished, hipStream_t s) {
  if (!logits || !ids || !last_ids || !row_len || !row_pos || !unfinished || rows <= 0 || vocab <= 0 ||
      max_step <= 0 || topk < 0 || (topk != 1 && !rng_state))
    return lsh_fail(LSH_ERR_INVALID, "lm_sample: bad arguments");
  if (topk == 0 && !(topp > 0.f && topp <= 1.f))
    return lsh_fail(LSH_ERR_INVALID, "lm_sample: topp must lie in (0, 1]");
  lm_sample_kernel<<<rows, 1024, 0, s>>>(logits, vocab, topk, topp, eos_id,
                                         static_cast<SampleState*>(rng_state), ids, max_step,
                                         last_ids, row_len, row_pos, unfinished);
  return lsh_check_launch("lm_sample_kernel");
}

}  // namespace lsh
