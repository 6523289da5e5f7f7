#include "sudevik.h"

#include "model_dir.h"
#include "sudevik_decoder.h"

namespace lightseq {
namespace hip {

Sudevik::Sudevik(const std::string model_dir, const ModelOptions& options) : DecoderLM(options) {
  const SudevikConfig config = SudevikConfig::parse(read_model_config(model_dir));
  open(model_dir, config.vocab,
       [&](const SafeTensors& file, const ModelOptions& o, hipStream_t stream) {
         return create_sudevik_stack(config, file, o.dtype == kFloat32, o.max_batch_size,
                                     o.max_step, stream);
       });
}

LSMODEL_REGISTER_ARCHITECTURE(Sudevik)

}  // namespace hip
}  // namespace lightseq
