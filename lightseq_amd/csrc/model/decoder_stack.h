// The layers of a decoder-only model over packed rows: one function runs a step, whether its sequences
// bring whole prompts, portions of them, or one token each.
#pragma once

#include "../lm_launch.h"
#include "model_util.h"

namespace lightseq {
namespace hip {

// One step on the device: rows of all sequences one after the other.
struct StepBatch {
  int rows = 0, n_seqs = 0;
  int max_n = 0;    // most rows of one sequence; 1: a decoding step, row r is sequence r
  int max_len = 0;  // no row's position is >= max_len
  const int *ids = nullptr, *row_slot = nullptr, *row_pos = nullptr;  // [rows]
  const lsh::SeqSpan* spans = nullptr;                                // [n_seqs]; unused if max_n == 1
  const int* want = nullptr;  // rows whose logits are asked for; null: every row
  int n_want = 0;
  int* zero_flag = nullptr;   // an int cleared on the way (what sampling counts in)
};

class DecoderStack {
 public:
  virtual ~DecoderStack() {}
  // room for steps of `rows` rows, of which n_want are asked for; true if buffers moved
  virtual bool reserve(int rows, int n_seqs, int n_want) = 0;
  // enqueues the step; the logits [n_want][vocab] are valid once the stream has passed it
  virtual const float* run(const StepBatch& b, const StepTaps& taps, int tap_step) = 0;
};

}  // namespace hip
}  // namespace lightseq
