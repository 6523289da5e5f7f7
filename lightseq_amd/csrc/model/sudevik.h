// "Sudevik": gated-delta and sliding-window-attention layers with mixtures of experts.
#pragma once

#include "decoder_lm.h"

namespace lightseq {
namespace hip {

class Sudevik : public DecoderLM {
 public:
  Sudevik(const std::string model_dir, const ModelOptions& options);
};

}  // namespace hip
}  // namespace lightseq
