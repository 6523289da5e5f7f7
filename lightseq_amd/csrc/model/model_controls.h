// Optional sides of a model behind the C ABI, implemented by the classes that have them: the controls
// of a generation loop, the debug aids of an encoder stack, and step-wise decoding of given tokens.
// model_capi.cpp finds them by dynamic_cast, so it depends on no model class.
#pragma once

#include <string>
#include <vector>

#include "model_util.h"

namespace lightseq {
namespace hip {

class GenerationControls {
 public:
  virtual ~GenerationControls() {}
  virtual StepTaps& step_taps() = 0;
  virtual void set_seed(unsigned long long seed) = 0;
  virtual void graph_mode(bool on) = 0;
  virtual const StepGraphs& graphs() const = 0;
  virtual const PhaseEvents& phases() const = 0;
  virtual int steps_run() const = 0;
  // per-step int8 logits (and sequences) of a run; false: this model keeps no such record
  virtual bool set_step_record(int8_t* /*logits*/, int* /*alive_seq*/, int /*max_steps*/) {
    return false;
  }
};

class EncoderControls {
 public:
  virtual ~EncoderControls() {}
  virtual void set_profiling(bool on) = 0;
  virtual std::string profile_json() = 0;
  virtual bool set_encoder_tap(int layer, const std::string& name, void* dst) = 0;
};

// Sequences that the caller feeds itself.  open() takes a place in the caches and states, close()
// gives it back; step() appends counts[i] tokens to sequence slots[i] (all entries are one batch)
// and writes the logits of the wanted rows (rows are numbered through the entries' tokens) to host
// memory [want][vocab].
class StepControls {
 public:
  virtual ~StepControls() {}
  virtual int open_sequence() = 0;
  virtual void close_sequence(int slot) = 0;
  virtual void step(const std::vector<int>& slots, const std::vector<int>& counts,
                    const std::vector<int>& tokens, const std::vector<int>& want,
                    float* host_logits) = 0;
  virtual int vocab_size() const = 0;
};

}  // namespace hip
}  // namespace lightseq
