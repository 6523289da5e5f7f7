// Sudevik's weights on the device.  Projections that read the same input are one matrix, so a layer's
// mixer starts with one product; linear weights have the type T of the activations, everything that
// is computed in float32 (norms, convolutions, gates' constants) is float.
#pragma once

#include "../float_device.h"
#include "model_util.h"
#include "safetensors.h"
#include "sudevik_config.h"

namespace lightseq {
namespace hip {

template <typename T>
struct SudevikLayerWeight {
  // layer norms ahead of (0, 2) and behind (1, 3) the mixer and the feed-forward
  DeviceBuffer<float> norm_w[4], norm_b[4];
  DeviceBuffer<T> in;   // rows q | k | v | g, then delta's b | a
  int q_col = 0, k_col = -1, v_col = -1, g_col = 0, t_cols = 0, in_cols = 0;
  DeviceBuffer<T> out;  // [width, heads * vdim]
  DeviceBuffer<float> q_norm, k_norm;                        // attention
  DeviceBuffer<float> conv, a_log, dt_bias, head_norm;       // delta
  DeviceBuffer<T> router, up, down;                          // up: [experts][2][ff][width]
  DeviceBuffer<float> router_b;
};

template <typename T>
struct SudevikWeight {
  DeviceBuffer<T> embed, head;
  DeviceBuffer<float> final_w, final_b;
  std::vector<SudevikLayerWeight<T>> layers;
  void load(const SudevikConfig& config, const SafeTensors& file, hipStream_t stream);
};

}  // namespace hip
}  // namespace lightseq
