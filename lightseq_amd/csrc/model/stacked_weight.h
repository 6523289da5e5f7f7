// Tensors of a safetensors file, converted to the type a kernel wants and stacked into one matrix.
#pragma once

#include "../float_device.h"
#include "model_util.h"
#include "safetensors.h"

namespace lightseq {
namespace hip {

using lsh::bf16_t;

inline float widen(uint16_t w) {
  const uint32_t u = (uint32_t)w << 16;
  float f;
  memcpy(&f, &u, 4);
  return f;
}

// n elements of a tensor as To, appended at dst
inline void convert(const SafeTensors::Tensor& t, float* dst) {
  const long n = t.count();
  if (t.dtype == "BF16") {
    const uint16_t* s = reinterpret_cast<const uint16_t*>(t.data);
    for (long i = 0; i < n; ++i) {
      uint16_t w;
      memcpy(&w, s + i, 2);
      dst[i] = widen(w);
    }
  } else if (t.dtype == "F32") {
    memcpy(dst, t.data, (size_t)n * 4);
  } else {
    throw std::runtime_error("weights must be bfloat16 or float32");
  }
}
inline void convert(const SafeTensors::Tensor& t, bf16_t* dst) {
  const long n = t.count();
  if (t.dtype == "BF16") {
    memcpy(static_cast<void*>(dst), t.data, (size_t)n * 2);
  } else if (t.dtype == "F32") {
    const uint8_t* s = t.data;
    for (long i = 0; i < n; ++i) {
      float f;
      memcpy(&f, s + 4 * i, 4);
      dst[i] = (bf16_t)f;
    }
  } else {
    throw std::runtime_error("weights must be bfloat16 or float32");
  }
}

template <typename E>
class Stacked {  // tensors one after the other, then one upload
 public:
  void add(const SafeTensors& f, const std::string& name, const std::vector<long>& shape) {
    const SafeTensors::Tensor& t = f.get(name, shape);
    const size_t at = host_.size();
    host_.resize(at + (size_t)t.count());
    convert(t, host_.data() + at);
  }
  // a matrix whose rows are filled up with zeros to `to` columns
  void add_rows(const SafeTensors& f, const std::string& name, long rows, long cols, long to) {
    std::vector<E> t((size_t)(rows * cols));
    convert(f.get(name, {rows, cols}), t.data());
    for (long r = 0; r < rows; ++r) {
      host_.insert(host_.end(), t.begin() + r * cols, t.begin() + (r + 1) * cols);
      add_zeros(to - cols);
    }
  }
  void add_zeros(long n) { host_.resize(host_.size() + (size_t)n); }
  DeviceBuffer<E> upload(hipStream_t s) {
    DeviceBuffer<E> d(host_.size());
    d.upload(host_.data(), host_.size(), s);
    CHECK_GPU_ERROR(hipStreamSynchronize(s));  // the host copy dies with this object
    return d;
  }

 private:
  std::vector<E> host_;
};

}  // namespace hip
}  // namespace lightseq
