// A decoder-only language model over packed rows and sequence slots, behind the LSModel interface:
// Infer() generates from a batch of prompts; the step interface feeds given tokens through the same
// layers, caches and states.  A design derives from it and supplies its layers (decoder_stack.h).
#pragma once

#include <functional>
#include <memory>

#include "decoder_stack.h"
#include "ls_model.h"
#include "model_controls.h"
#include "safetensors.h"
#include "sequence_cache.h"

namespace lightseq {
namespace hip {

class DecoderLM : public LSModel, public GenerationControls, public StepControls {
 public:
  ~DecoderLM();

  void Infer() override;
  void benchmark_mode(bool is_benchmark) override { _is_benchmark = is_benchmark; }
  void* get_stream() override { return stream_.get(); }

  StepTaps& step_taps() override { return _taps; }
  void set_seed(unsigned long long seed) override;
  void graph_mode(bool on) override { _use_graphs = on; }
  const StepGraphs& graphs() const override { return _graphs; }
  const PhaseEvents& phases() const override { return _phases; }
  int steps_run() const override { return _steps_run; }

  int open_sequence() override { return _slots->open(); }
  void close_sequence(int slot) override { _slots->close(slot); }
  void step(const std::vector<int>& slots, const std::vector<int>& counts,
            const std::vector<int>& tokens, const std::vector<int>& want,
            float* host_logits) override;
  int vocab_size() const override { return _vocab; }

 protected:
  using BuildStack = std::function<std::unique_ptr<DecoderStack>(const SafeTensors&,
                                                                 const ModelOptions&, hipStream_t)>;
  explicit DecoderLM(const ModelOptions& options);  // checks the options; touches no GPU
  // the rest of the construction, once the design has read its config.json
  void open(const std::string& model_dir, int vocab, const BuildStack& build);

 private:
  const float* enqueue(const std::vector<int>& slots, const std::vector<int>& counts,
                       const std::vector<int>& tokens, const std::vector<int>& want);
  void sample(const float* logits, int batch);
  int generate(const std::vector<int>& slots, std::vector<int>& lengths,
               const std::vector<int>& tokens);

  // owners first: the stream outlives everything that was enqueued on it
  StreamOwner stream_;
  ModelOptions _opt;
  int _vocab = 0;
  std::unique_ptr<DecoderStack> _stack;
  std::unique_ptr<SequenceSlots> _slots;
  DeviceBuffer<int> d_input_, d_result_;
  int *_p_d_token_id = nullptr, *_p_d_result = nullptr;
  DeviceBuffer<int> _batch;  // a step's ids, slots, positions, spans and wanted rows
  int* _h_batch = nullptr;   // the same, pinned
  size_t _batch_ints = 0;
  // generation: device state of the rows
  DeviceBuffer<int> _ids, _last_ids, _row_slot, _row_pos, _row_len, _unfinished;
  DeviceBuffer<long long> _rng;
  int* _h_unfinished = nullptr;  // pinned
  StepTaps _taps;
  StepGraphs _graphs;
  PhaseEvents _phases;
  bool _is_benchmark = false, _use_graphs = false;
  int _steps_run = 0;
};

}  // namespace hip
}  // namespace lightseq
