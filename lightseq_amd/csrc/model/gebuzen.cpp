#include "gebuzen.h"

#include "model_dir.h"
#include "gebuzen_decoder.h"

namespace lightseq {
namespace hip {

Gebuzen::Gebuzen(const std::string model_dir, const ModelOptions& options) : DecoderLM(options) {
  const GebuzenConfig config = GebuzenConfig::parse(read_model_config(model_dir));
  open(model_dir, config.vocab,
       [&](const SafeTensors& file, const ModelOptions& o, hipStream_t stream) {
         return create_gebuzen_stack(config, file, o.dtype == kFloat32, o.max_batch_size,
                                     o.max_step, stream);
       });
}

LSMODEL_REGISTER_ARCHITECTURE(Gebuzen)

}  // namespace hip
}  // namespace lightseq
