#pragma once

#include <string>

#include "json.h"

namespace lightseq {
namespace hip {

Json read_model_config(const std::string& model_dir);  // <model_dir>/config.json

}  // namespace hip
}  // namespace lightseq
