// What config.json says about a Gebuzen decoder: an ordered list of layers, each two mixers side by
// side (attention in chunks whose values are its keys, gated linear attention) followed by an optional
// feed-forward; a run of layers may be passed through several times.
#pragma once

#include <vector>

#include "json.h"

namespace lightseq {
namespace hip {

struct GebuzenLayerConfig {
  // left: attention
  int heads = 0, kv_heads = 0, dim = 0;
  double scale = 1;
  int chunk = 0;  // 0: every earlier token
  // right: gated linear attention
  int gla_heads = 0, gla_dim = 0, gla_vdim = 0;
  double tau = 1;
  int ff = 0;  // 0: no feed-forward
};

// One run through a layer.
struct GebuzenLayerRun {
  int layer = 0;
  int step = -1;               // row of the step vectors that is added ahead of it; -1: none
  bool again = false;          // the embedding output is added ahead of it
};

struct GebuzenConfig {
  int vocab = 0, width = 0;
  double eps = 0, residual_mult = 1, logit_scale = 1;
  std::vector<GebuzenLayerConfig> layers;
  int loop_start = 0, loop_stop = 0, loop_times = 0;  // loop_times == 0: no loop
  static GebuzenConfig parse(const Json& config);
  std::vector<GebuzenLayerRun> runs() const;  // in their order
};

}  // namespace hip
}  // namespace lightseq
