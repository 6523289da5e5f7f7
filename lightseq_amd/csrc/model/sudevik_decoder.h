// The layers of a Sudevik decoder.
#pragma once

#include <memory>

#include "decoder_stack.h"
#include "safetensors.h"
#include "sudevik_config.h"

namespace lightseq {
namespace hip {

std::unique_ptr<DecoderStack> create_sudevik_stack(const SudevikConfig& config,
                                                   const SafeTensors& file, bool float32, int slots,
                                                   int max_step, hipStream_t stream);

}  // namespace hip
}  // namespace lightseq
