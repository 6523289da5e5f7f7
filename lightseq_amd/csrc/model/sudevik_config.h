// What config.json says about a Sudevik decoder: an ordered list of layers, each an attention or a
// gated-delta mixer followed by an optional mixture of experts.
#pragma once

#include <string>
#include <vector>

#include "json.h"

namespace lightseq {
namespace hip {

struct RotaryConfig {
  int dims = 0;  // 0: no rotation
  double base = 1;
  bool scaled = false;  // YaRN
  double factor = 1, original = 1, fast = 1, slow = 1;
  bool operator==(const RotaryConfig& o) const {
    return dims == o.dims && base == o.base && scaled == o.scaled && factor == o.factor &&
           original == o.original && fast == o.fast && slow == o.slow;
  }
  // angle per position of every pair, and the factor on cosine and sine
  std::vector<double> frequencies(double* magnitude) const;
};

struct SudevikLayerConfig {
  bool attention = false;  // else delta
  int heads = 0, kv_heads = 0, dim = 0, vdim = 0;
  // attention
  RotaryConfig rot;
  double scale = 1;
  int window = 0;  // 0: every earlier token
  int keep_first = 0;
  int kv_from = -1;  // the layer whose keys and values are used; -1: its own
  // delta
  int taps = 0;
  // mixture of experts; experts == 0: none
  int experts = 0, top = 0, ff = 0;
};

struct SudevikConfig {
  int vocab = 0, width = 0;
  double eps = 0;
  std::vector<SudevikLayerConfig> layers;
  static SudevikConfig parse(const Json& config);
};

}  // namespace hip
}  // namespace lightseq
