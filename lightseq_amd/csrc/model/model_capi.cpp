// extern "C" wrapper of the LSModel interface: exceptions -> status codes.
#include <string.h>

#include <memory>

#include "../../../include/lightseq_model.h"
#include "../ls_launch.h"
#include "ls_model.h"
#include "model_controls.h"

using lightseq::hip::EncoderControls;
using lightseq::hip::GenerationControls;
using lightseq::hip::LSModel;
using lightseq::hip::LSModelFactory;
using lightseq::hip::ModelOptions;
using lightseq::hip::StepControls;

struct ls_model {
  std::unique_ptr<LSModel> impl;
  std::string name_buf;
};

namespace {

template <typename F>
int guarded(F&& f) {
  try {
    f();
    return LSH_OK;
  } catch (const std::exception& e) {
    return lsh::lsh_fail(LSH_ERR_INVALID, e.what());
  } catch (...) {
    return lsh::lsh_fail(LSH_ERR_INVALID, "unknown C++ exception");
  }
}

int copy_shape(const std::vector<int>& v, int* shape, int* ndim) {
  if (!shape || !ndim) return lsh::lsh_fail(LSH_ERR_INVALID, "null shape pointer");
  if (v.size() > LS_MAX_DIMS) return lsh::lsh_fail(LSH_ERR_INVALID, "too many dimensions");
  *ndim = (int)v.size();
  for (size_t i = 0; i < v.size(); ++i) shape[i] = v[i];
  return LSH_OK;
}

// an optional side of a model, or nullptr
template <typename Side>
Side* side_of(ls_model* model) {
  return dynamic_cast<Side*>(model->impl.get());
}

#define NEED_MODEL(m) \
  if (!(m) || !(m)->impl) return lsh::lsh_fail(LSH_ERR_INVALID, "null model handle")

}  // namespace

extern "C" {

int ls_model_create(const char* class_name, const char* weight_path, int max_batch_size,
                    ls_model** model) {
  if (!class_name || !weight_path || !model)
    return lsh::lsh_fail(LSH_ERR_INVALID, "ls_model_create: null argument");
  *model = nullptr;
  return guarded([&] {
    LSModel* p = LSModelFactory::GetInstance().CreateModel(class_name, weight_path, max_batch_size);
    *model = new ls_model{std::unique_ptr<LSModel>(p), {}};
  });
}

int ls_model_destroy(ls_model* model) {
  if (!model) return LSH_OK;
  return guarded([&] { delete model; });
}

int ls_model_infer(ls_model* model) {
  NEED_MODEL(model);
  return guarded([&] { model->impl->Infer(); });
}

int ls_model_set_input_ptr(ls_model* model, int index, void* input_ptr) {
  NEED_MODEL(model);
  return guarded([&] { model->impl->set_input_ptr(index, input_ptr); });
}

int ls_model_set_input_shape(ls_model* model, int index, const int* shape, int ndim) {
  NEED_MODEL(model);
  if (!shape || ndim < 0 || ndim > LS_MAX_DIMS)
    return lsh::lsh_fail(LSH_ERR_INVALID, "ls_model_set_input_shape: bad shape");
  return guarded([&] { model->impl->set_input_shape(index, std::vector<int>(shape, shape + ndim)); });
}

int ls_model_get_input_max_shape(ls_model* model, int index, int* shape, int* ndim) {
  NEED_MODEL(model);
  int rc = LSH_OK;
  int g = guarded([&] { rc = copy_shape(model->impl->get_input_max_shape(index), shape, ndim); });
  return g ? g : rc;
}

int ls_model_get_input_size(ls_model* model, int* count) {
  NEED_MODEL(model);
  if (!count) return lsh::lsh_fail(LSH_ERR_INVALID, "null pointer");
  *count = model->impl->get_input_size();
  return LSH_OK;
}

int ls_model_get_input_name(ls_model* model, int index, const char** name) {
  NEED_MODEL(model);
  if (!name) return lsh::lsh_fail(LSH_ERR_INVALID, "null pointer");
  return guarded([&] {
    model->name_buf = model->impl->get_input_name(index);
    *name = model->name_buf.c_str();
  });
}

int ls_model_get_input_dtype(ls_model* model, int index, int* dtype) {
  NEED_MODEL(model);
  if (!dtype) return lsh::lsh_fail(LSH_ERR_INVALID, "null pointer");
  return guarded([&] { *dtype = (int)model->impl->get_input_dtype(index); });
}

int ls_model_set_output_ptr(ls_model* model, int index, void* output_ptr) {
  NEED_MODEL(model);
  return guarded([&] { model->impl->set_output_ptr(index, output_ptr); });
}

int ls_model_get_output_ptr(ls_model* model, int index, const void** output_ptr) {
  NEED_MODEL(model);
  if (!output_ptr) return lsh::lsh_fail(LSH_ERR_INVALID, "null pointer");
  return guarded([&] { *output_ptr = model->impl->get_output_ptr(index); });
}

int ls_model_get_output_size(ls_model* model, int* count) {
  NEED_MODEL(model);
  if (!count) return lsh::lsh_fail(LSH_ERR_INVALID, "null pointer");
  *count = model->impl->get_output_size();
  return LSH_OK;
}

int ls_model_get_output_name(ls_model* model, int index, const char** name) {
  NEED_MODEL(model);
  if (!name) return lsh::lsh_fail(LSH_ERR_INVALID, "null pointer");
  return guarded([&] {
    model->name_buf = model->impl->get_output_name(index);
    *name = model->name_buf.c_str();
  });
}

int ls_model_get_output_shape(ls_model* model, int index, int* shape, int* ndim) {
  NEED_MODEL(model);
  int rc = LSH_OK;
  int g = guarded([&] { rc = copy_shape(model->impl->get_output_shape(index), shape, ndim); });
  return g ? g : rc;
}

int ls_model_get_output_max_shape(ls_model* model, int index, int* shape, int* ndim) {
  NEED_MODEL(model);
  int rc = LSH_OK;
  int g = guarded([&] { rc = copy_shape(model->impl->get_output_max_shape(index), shape, ndim); });
  return g ? g : rc;
}

int ls_model_get_output_dtype(ls_model* model, int index, int* dtype) {
  NEED_MODEL(model);
  if (!dtype) return lsh::lsh_fail(LSH_ERR_INVALID, "null pointer");
  return guarded([&] { *dtype = (int)model->impl->get_output_dtype(index); });
}

int ls_model_benchmark_mode(ls_model* model, int is_benchmark) {
  NEED_MODEL(model);
  return guarded([&] { model->impl->benchmark_mode(is_benchmark != 0); });
}

int ls_model_get_stream(ls_model* model, lsh_stream_t* stream) {
  NEED_MODEL(model);
  if (!stream) return lsh::lsh_fail(LSH_ERR_INVALID, "null pointer");
  *stream = reinterpret_cast<lsh_stream_t>(model->impl->get_stream());
  return LSH_OK;
}

#define NEED_SIDE(var, Side, message)            \
  Side* var = side_of<Side>(model);              \
  if (!var) return lsh::lsh_fail(LSH_ERR_UNSUPPORTED, message)
#define NO_GENERATION "this model has no generation steps"

int ls_model_set_profiling(ls_model* model, int on) {
  NEED_MODEL(model);
  NEED_SIDE(enc, EncoderControls, "this model has no profiled encoder stack");
  return guarded([&] { enc->set_profiling(on != 0); });
}

int ls_model_get_profile(ls_model* model, char* buf, int capacity) {
  NEED_MODEL(model);
  NEED_SIDE(enc, EncoderControls, "this model has no profiled encoder stack");
  if (!buf || capacity <= 0) return lsh::lsh_fail(LSH_ERR_INVALID, "null buffer");
  const std::string out = enc->profile_json();
  if ((int)out.size() + 1 > capacity) return lsh::lsh_fail(LSH_ERR_INVALID, "buffer too small");
  memcpy(buf, out.c_str(), out.size() + 1);
  return LSH_OK;
}

int ls_model_set_tap(ls_model* model, int layer, const char* name, void* dst) {
  NEED_MODEL(model);
  if (!name) return lsh::lsh_fail(LSH_ERR_INVALID, "null pointer");
  // "dec.<name>": an intermediate of a generation step (layer `layer`, at the step given to
  // ls_model_set_tap_step)
  if (!strncmp(name, "dec.", 4)) {
    NEED_SIDE(gen, GenerationControls, NO_GENERATION);
    gen->step_taps().set(layer, name + 4, dst);
    return LSH_OK;
  }
  NEED_SIDE(enc, EncoderControls, "this model has no tapped encoder stack");
  if (!enc->set_encoder_tap(layer, name, dst))
    return lsh::lsh_fail(LSH_ERR_INVALID, "unknown tap name");
  return LSH_OK;
}

int ls_model_set_tap_step(ls_model* model, int step) {
  NEED_MODEL(model);
  NEED_SIDE(gen, GenerationControls, NO_GENERATION);
  gen->step_taps().set_step(step);
  return LSH_OK;
}

int ls_model_set_step_record(ls_model* model, int8_t* logits, int* alive_seq, int max_steps) {
  NEED_MODEL(model);
  if (max_steps < 0) return lsh::lsh_fail(LSH_ERR_INVALID, "negative max_steps");
  NEED_SIDE(gen, GenerationControls, NO_GENERATION);
  if (!gen->set_step_record(logits, alive_seq, max_steps))
    return lsh::lsh_fail(LSH_ERR_UNSUPPORTED,
                         "step records are a debug aid of QuantTransformer and QuantGpt");
  return LSH_OK;
}

int ls_model_set_graph_mode(ls_model* model, int on) {
  NEED_MODEL(model);
  NEED_SIDE(gen, GenerationControls, NO_GENERATION);
  gen->graph_mode(on != 0);
  return LSH_OK;
}

int ls_model_set_seed(ls_model* model, unsigned long long seed) {
  NEED_MODEL(model);
  NEED_SIDE(gen, GenerationControls, NO_GENERATION);
  return guarded([&] { gen->set_seed(seed); });
}

int ls_model_get_graph_stats(ls_model* model, int* captured, long long* replayed) {
  NEED_MODEL(model);
  if (!captured || !replayed) return lsh::lsh_fail(LSH_ERR_INVALID, "null pointer");
  NEED_SIDE(gen, GenerationControls, NO_GENERATION);
  *captured = gen->graphs().captured();
  *replayed = gen->graphs().replayed();
  return LSH_OK;
}

int ls_model_get_graph_nodes(ls_model* model, int* nodes) {
  NEED_MODEL(model);
  if (!nodes) return lsh::lsh_fail(LSH_ERR_INVALID, "null pointer");
  NEED_SIDE(gen, GenerationControls, NO_GENERATION);
  *nodes = gen->graphs().last_graph_nodes();
  return LSH_OK;
}

int ls_model_get_phase_times(ls_model* model, float* prepare_ms, float* steps_ms, int* steps) {
  NEED_MODEL(model);
  if (!prepare_ms || !steps_ms || !steps) return lsh::lsh_fail(LSH_ERR_INVALID, "null pointer");
  NEED_SIDE(gen, GenerationControls, NO_GENERATION);
  bool have = false;
  const int rc = guarded([&] { have = gen->phases().times(prepare_ms, steps_ms, steps); });
  if (rc != LSH_OK) return rc;
  if (!have) return lsh::lsh_fail(LSH_ERR_INVALID, "no generation run has completed yet");
  return LSH_OK;
}

int ls_model_get_steps_run(ls_model* model, int* steps) {
  NEED_MODEL(model);
  if (!steps) return lsh::lsh_fail(LSH_ERR_INVALID, "null pointer");
  NEED_SIDE(gen, GenerationControls, NO_GENERATION);
  *steps = gen->steps_run();
  return LSH_OK;
}

// ---- models in a folder, step-wise decoding ------------------------------------------------
void ls_model_default_options(ls_model_options* o) {
  if (!o) return;
  const ModelOptions d;
  o->max_batch_size = d.max_batch_size;
  o->max_step = d.max_step;
  o->dtype = (int)d.dtype;
  o->topk = d.topk;
  o->topp = d.topp;
  o->eos_id = d.eos_id;
  o->padding_id = d.padding_id;
  o->extra_decode_length = d.extra_decode_length;
}

int ls_model_create_from_dir(const char* model_dir, const ls_model_options* o, ls_model** model) {
  if (!model_dir || !model)
    return lsh::lsh_fail(LSH_ERR_INVALID, "ls_model_create_from_dir: null argument");
  *model = nullptr;
  return guarded([&] {
    ModelOptions opt;
    if (o) {
      opt.max_batch_size = o->max_batch_size;
      opt.max_step = o->max_step;
      opt.dtype = (lightseq::hip::DataType)o->dtype;
      opt.topk = o->topk;
      opt.topp = o->topp;
      opt.eos_id = o->eos_id;
      opt.padding_id = o->padding_id;
      opt.extra_decode_length = o->extra_decode_length;
    }
    LSModel* p = LSModelFactory::GetInstance().CreateFromDirectory(model_dir, opt);
    *model = new ls_model{std::unique_ptr<LSModel>(p), {}};
  });
}

#define NO_STEPS "this model does not decode step by step"

int ls_model_get_vocab_size(ls_model* model, int* size) {
  NEED_MODEL(model);
  if (!size) return lsh::lsh_fail(LSH_ERR_INVALID, "null pointer");
  NEED_SIDE(st, StepControls, NO_STEPS);
  *size = st->vocab_size();
  return LSH_OK;
}

int ls_model_open_sequence(ls_model* model, int* slot) {
  NEED_MODEL(model);
  if (!slot) return lsh::lsh_fail(LSH_ERR_INVALID, "null pointer");
  NEED_SIDE(st, StepControls, NO_STEPS);
  return guarded([&] { *slot = st->open_sequence(); });
}

int ls_model_close_sequence(ls_model* model, int slot) {
  NEED_MODEL(model);
  NEED_SIDE(st, StepControls, NO_STEPS);
  return guarded([&] { st->close_sequence(slot); });
}

int ls_model_step(ls_model* model, int entries, const int* slots, const int* counts,
                  const int* tokens, int n_want, const int* want_rows, float* logits) {
  NEED_MODEL(model);
  NEED_SIDE(st, StepControls, NO_STEPS);
  if (entries <= 0 || !slots || !counts || !tokens || n_want < 0 ||
      (n_want > 0 && (!want_rows || !logits)))
    return lsh::lsh_fail(LSH_ERR_INVALID, "ls_model_step: bad arguments");
  return guarded([&] {
    long rows = 0;
    for (int i = 0; i < entries; ++i) rows += counts[i] > 0 ? counts[i] : 0;
    st->step(std::vector<int>(slots, slots + entries), std::vector<int>(counts, counts + entries),
             std::vector<int>(tokens, tokens + rows),
             std::vector<int>(want_rows, want_rows + n_want), logits);
  });
}

}  // extern "C"
