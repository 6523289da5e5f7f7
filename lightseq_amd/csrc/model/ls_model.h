// C++ model interface of the library: the same abstract class, factory and
// registration macro as the reference's lightseq::cuda::LSModel
// (lightseq/inference/pywrapper/model_base.h:12-148), in namespace lightseq::hip.
// Errors are C++ exceptions (std::runtime_error), as in the reference; the C ABI in
// include/lightseq_model.h turns them into status codes.
#pragma once

#include <map>
#include <stdexcept>
#include <string>
#include <vector>

namespace lightseq {
namespace hip {

enum DataType {
  kNotSupported = 0, kFloat32 = 1, kInt32 = 2, kInt64 = 3, kFloat16 = 4, kInt8 = 5, kInt16 = 6,
  kByte = 7, kUInt8 = 8, kUInt16 = 9, kUInt32 = 10, kUInt64 = 11, kFloat64 = 12,
  kBFloat16 = 13  // not in the reference
};

// One input or output of a model: what the accessor functions of LSModel answer from.  `slot`
// is where the model keeps the device pointer of this tensor (inside its encoder / decoder).
struct IoSlot {
  DataType dtype = kNotSupported;
  std::vector<int> max_shape;
  void** slot = nullptr;
};

class LSModel {
 public:
  LSModel(std::vector<std::string> input_names, std::vector<std::string> output_names)
      : kInputNames(std::move(input_names)), kOutputNames(std::move(output_names)) {
    input_shapes_.resize(kInputNames.size());
    output_shapes_.resize(kOutputNames.size());
    inputs_.resize(kInputNames.size());
    outputs_.resize(kOutputNames.size());
  }
  virtual ~LSModel() {}
  virtual void Infer() = 0;

  // The accessors below are answered from the descriptor table that the model's constructor
  // fills (describe_input / describe_output); a model overrides none of them.
  virtual void set_input_ptr(int index, void* input_ptr) { *slot_of(inputs_, index, "input").slot = input_ptr; }
  void set_input_shape(int index, std::vector<int> shape) {
    input_shapes_.at(index) = std::move(shape);
  }
  virtual std::vector<int> get_input_max_shape(int index) {
    return slot_of(inputs_, index, "input").max_shape;
  }
  std::string get_input_name(int index) { return kInputNames.at(index); }
  int get_input_size() { return (int)kInputNames.size(); }
  virtual DataType get_input_dtype(int index) { return slot_of(inputs_, index, "input").dtype; }

  virtual void set_output_ptr(int index, void* output_ptr) {
    *slot_of(outputs_, index, "output").slot = output_ptr;
  }
  virtual const void* get_output_ptr(int index) { return *slot_of(outputs_, index, "output").slot; }
  std::string get_output_name(int index) { return kOutputNames.at(index); }
  int get_output_size() { return (int)kOutputNames.size(); }
  std::vector<int> get_output_shape(int index) { return output_shapes_.at(index); }
  virtual std::vector<int> get_output_max_shape(int index) {
    return slot_of(outputs_, index, "output").max_shape;
  }
  virtual DataType get_output_dtype(int index) { return slot_of(outputs_, index, "output").dtype; }

  virtual void benchmark_mode(bool is_benchmark) = 0;

  // Not in the reference: the HIP stream the model launches on (for event timing).
  virtual void* get_stream() = 0;

 protected:
  void set_output_shape(int index, std::vector<int> shape) {
    output_shapes_.at(index) = std::move(shape);
  }
  template <typename T>
  void describe_input(int index, DataType dtype, std::vector<int> max_shape, T** slot) {
    inputs_.at(index) = IoSlot{dtype, std::move(max_shape), (void**)slot};
  }
  template <typename T>
  void describe_output(int index, DataType dtype, std::vector<int> max_shape, T** slot) {
    outputs_.at(index) = IoSlot{dtype, std::move(max_shape), (void**)slot};
  }
  const std::vector<std::string> kInputNames;
  const std::vector<std::string> kOutputNames;
  std::vector<std::vector<int>> input_shapes_;
  std::vector<std::vector<int>> output_shapes_;

 private:
  static IoSlot& slot_of(std::vector<IoSlot>& table, int index, const char* what) {
    if (index < 0 || index >= (int)table.size() || table[index].slot == nullptr)
      throw std::runtime_error(std::string("invalid ") + what + " index");
    return table[index];
  }
  std::vector<IoSlot> inputs_, outputs_;
};

typedef LSModel* (*LSModelConstructor)(const std::string, const int);

// What a model folder (config.json + weights) does not say about serving it.
struct ModelOptions {
  int max_batch_size = 8;
  int max_step = 2048;          // positions a sequence can have
  DataType dtype = kBFloat16;   // or kFloat32
  int topk = 1;                 // 1: greedy; > 1: top-k; 0: top-p
  float topp = 0.75f;
  int eos_id = -1;              // -1: none
  int padding_id = -1;          // right padding of short prompts, and of short results
  int extra_decode_length = 64; // tokens generated after the longest prompt
};
typedef LSModel* (*LSModelDirConstructor)(const std::string, const ModelOptions&);

class LSModelFactory {
 public:
  static LSModelFactory& GetInstance() {
    static LSModelFactory factory;
    return factory;
  }
  void ModelRegister(std::string class_name, LSModelConstructor obj) {
    if (obj) object_map_.insert({class_name, obj});
  }
  LSModel* CreateModel(std::string class_name, const std::string weight_path,
                       const int max_batch_size) {
    auto iter = object_map_.find(class_name);
    if (iter == object_map_.end()) throw std::runtime_error("Model not supported");
    return iter->second(weight_path, max_batch_size);
  }
  // Models in folders are registered under the "architecture" of their config.json.
  void ArchitectureRegister(std::string architecture, LSModelDirConstructor obj) {
    if (obj) dir_map_.insert({architecture, obj});
  }
  LSModel* CreateFromDirectory(const std::string model_dir, const ModelOptions& options);

 private:
  LSModelFactory() {}
  std::map<std::string, LSModelConstructor> object_map_;
  std::map<std::string, LSModelDirConstructor> dir_map_;
};

class Reflector {
 public:
  Reflector(std::string name, LSModelConstructor obj) {
    LSModelFactory::GetInstance().ModelRegister(name, obj);
  }
  Reflector(std::string architecture, LSModelDirConstructor obj) {
    LSModelFactory::GetInstance().ArchitectureRegister(architecture, obj);
  }
};

#define LSMODEL_REGISTER(className)                                                         \
  LSModel* create_object_##className(const std::string weight_path,                         \
                                     const int max_batch_size) {                            \
    return new className(weight_path, max_batch_size);                                      \
  }                                                                                         \
  Reflector reflector_##className(#className, create_object_##className);

// The class under its name (weight_path: the folder, default options) and as the architecture of
// that name.
#define LSMODEL_REGISTER_ARCHITECTURE(className)                                            \
  LSModel* create_object_##className(const std::string path, const int max_batch_size) {    \
    ModelOptions options;                                                                   \
    options.max_batch_size = max_batch_size;                                                \
    return new className(path, options);                                                    \
  }                                                                                         \
  LSModel* create_architecture_##className(const std::string path,                          \
                                           const ModelOptions& options) {                   \
    return new className(path, options);                                                    \
  }                                                                                         \
  Reflector reflector_##className(#className, create_object_##className);                   \
  Reflector reflector_architecture_##className(#className, create_architecture_##className);

}  // namespace hip
}  // namespace lightseq
