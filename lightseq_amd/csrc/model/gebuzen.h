// "Gebuzen": chunked attention and gated linear attention side by side in every layer, dense
// feed-forwards, and a run of layers that is passed through several times.
#pragma once

#include "decoder_lm.h"

namespace lightseq {
namespace hip {

class Gebuzen : public DecoderLM {
 public:
  Gebuzen(const std::string model_dir, const ModelOptions& options);
};

}  // namespace hip
}  // namespace lightseq
