// The layers of a Gebuzen decoder.
#pragma once

#include <memory>

#include "decoder_stack.h"
#include "gebuzen_config.h"
#include "safetensors.h"

namespace lightseq {
namespace hip {

std::unique_ptr<DecoderStack> create_gebuzen_stack(const GebuzenConfig& config,
                                                   const SafeTensors& file, bool float32, int slots,
                                                   int max_step, hipStream_t stream);

}  // namespace hip
}  // namespace lightseq
