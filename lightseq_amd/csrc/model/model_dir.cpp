// Models in folders: the "architecture" of config.json chooses the class.
#include "model_dir.h"

#include <fstream>
#include <sstream>

#include "ls_model.h"

namespace lightseq {
namespace hip {

Json read_model_config(const std::string& model_dir) {
  const std::string path = model_dir + "/config.json";
  std::ifstream in(path, std::ios::binary);
  if (!in) throw std::runtime_error("File " + path + " not found.");
  std::stringstream text;
  text << in.rdbuf();
  return Json::parse(text.str());
}

LSModel* LSModelFactory::CreateFromDirectory(const std::string model_dir,
                                             const ModelOptions& options) {
  const std::string arch = read_model_config(model_dir).at("architecture").string();
  auto iter = dir_map_.find(arch);
  if (iter == dir_map_.end()) throw std::runtime_error("Model not supported: " + arch);
  return iter->second(model_dir, options);
}

}  // namespace hip
}  // namespace lightseq
