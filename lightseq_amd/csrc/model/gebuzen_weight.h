// Gebuzen's weights on the device.  Everything that reads a layer's mixer input is one matrix (the
// projections of both mixers, then the narrow product of the decays, whose result stays float);
// linear weights have the type T of the activations, norms, biases, sinks and the decays' second
// product are float.
#pragma once

#include "../float_device.h"
#include "gebuzen_config.h"
#include "model_util.h"
#include "safetensors.h"

namespace lightseq {
namespace hip {

template <typename T>
struct GebuzenLayerWeight {
  DeviceBuffer<float> norm1, norm2;
  // columns of `in`: left q | k, right q | k | v | g (each from a multiple of 8 on), then the narrow
  // product, padded with zeros to `rank`
  DeviceBuffer<T> in;
  DeviceBuffer<float> in_bias;
  int q_col = 0, k_col = 0, gq_col = 0, gk_col = 0, gv_col = 0, gg_col = 0;
  int t_cols = 0, in_cols = 0, rank = 0;
  DeviceBuffer<float> sink;
  DeviceBuffer<float> a2, a2_bias, head_norm;
  DeviceBuffer<T> left_o, right_o;
  DeviceBuffer<float> left_norm, right_norm;
  DeviceBuffer<T> up, down;  // up: [2][ff][width]
};

template <typename T>
struct GebuzenWeight {
  DeviceBuffer<T> embed, head;
  DeviceBuffer<float> final_norm;
  DeviceBuffer<float> loop_step;  // [times][width]
  std::vector<GebuzenLayerWeight<T>> layers;
  void load(const GebuzenConfig& config, const SafeTensors& file, hipStream_t stream);
};

}  // namespace hip
}  // namespace lightseq
