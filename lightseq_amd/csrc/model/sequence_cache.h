// What live sequences leave behind between steps, by slot: keys and values of fixed stride
// [slot][kv_head][max_step][pad], recurrent states and the last inputs of short convolutions.  A
// slot is given out when a sequence opens and taken back when it closes; nothing is cleared in
// between, because kernels read only what the same sequence has written (positions below its
// length; a state only from its second token on).
#pragma once

#include <map>
#include <vector>

#include "model_util.h"

namespace lightseq {
namespace hip {

class SequenceSlots {
 public:
  SequenceSlots(int slots, int max_step) : length_(slots, -1), max_step_(max_step) {
    for (int i = slots - 1; i >= 0; --i) free_.push_back(i);
  }
  int open() {
    if (free_.empty()) throw std::runtime_error("no free sequence slot (max_batch_size is live)");
    const int s = free_.back();
    free_.pop_back();
    length_[s] = 0;
    return s;
  }
  void close(int slot) {
    check(slot);
    length_[slot] = -1;
    free_.push_back(slot);
  }
  int length(int slot) const {
    check(slot);
    return length_[slot];
  }
  void advance(int slot, int n) {
    check(slot);
    if (length_[slot] + n > max_step_) throw std::runtime_error("sequence longer than max_step");
    length_[slot] += n;
  }
  int slots() const { return (int)length_.size(); }
  int max_step() const { return max_step_; }

 private:
  void check(int slot) const {
    if (slot < 0 || slot >= (int)length_.size() || length_[slot] < 0)
      throw std::runtime_error("not an open sequence");
  }
  std::vector<int> length_, free_;  // length -1: free
  const int max_step_;
};

// Storage of one layer; T is the type of the activations.
template <typename T>
struct LayerCache {
  DeviceBuffer<T> k, v;         // attention with keys of its own (no v: the values are the keys)
  DeviceBuffer<T> conv;         // delta layers: ring of the convolutions' inputs
  DeviceBuffer<float> state;    // recurrent layers: delta [slot][heads][dim][vdim], gated linear
                                // attention [slot][heads][vdim][dim]
};

}  // namespace hip
}  // namespace lightseq
