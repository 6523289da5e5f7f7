// A safetensors file mapped into memory: an 8-byte little-endian length, that many bytes of JSON
// (name -> dtype, shape, data_offsets), then the data.
#pragma once

#include <fcntl.h>
#include <string.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <cstdint>

#include "json.h"

namespace lightseq {
namespace hip {

class SafeTensors {
 public:
  struct Tensor {
    std::string dtype;
    std::vector<long> shape;
    const uint8_t* data = nullptr;
    long count() const {
      long n = 1;
      for (long d : shape) n *= d;
      return n;
    }
  };

  explicit SafeTensors(const std::string& path) {
    const int fd = open(path.c_str(), O_RDONLY | O_CLOEXEC);
    if (fd < 0) throw std::runtime_error("File " + path + " not found.");
    struct stat st;
    if (fstat(fd, &st) != 0 || st.st_size < 8) {
      close(fd);
      throw std::runtime_error(path + ": not a safetensors file");
    }
    size_ = (size_t)st.st_size;
    map_ = mmap(nullptr, size_, PROT_READ, MAP_PRIVATE, fd, 0);
    close(fd);
    if (map_ == MAP_FAILED) {
      map_ = nullptr;
      throw std::runtime_error(path + ": cannot be mapped");
    }
    try {
      index(path);
    } catch (...) {
      munmap(map_, size_);
      throw;
    }
  }
  SafeTensors(const SafeTensors&) = delete;
  SafeTensors& operator=(const SafeTensors&) = delete;
  ~SafeTensors() {
    if (map_) munmap(map_, size_);
  }

  bool has(const std::string& name) const { return tensors_.count(name) != 0; }
  const Tensor& get(const std::string& name) const {
    auto it = tensors_.find(name);
    if (it == tensors_.end()) throw std::runtime_error("tensor '" + name + "' is missing");
    return it->second;
  }
  // the tensor, with the shape it must have
  const Tensor& get(const std::string& name, const std::vector<long>& shape) const {
    const Tensor& t = get(name);
    if (t.shape != shape) {
      std::string m = "tensor '" + name + "' has the shape [";
      for (long d : t.shape) m += std::to_string(d) + " ";
      m += "], expected [";
      for (long d : shape) m += std::to_string(d) + " ";
      throw std::runtime_error(m + "]");
    }
    return t;
  }

 private:
  void index(const std::string& path) {
    const uint8_t* p = static_cast<const uint8_t*>(map_);
    uint64_t n = 0;
    for (int i = 7; i >= 0; --i) n = n << 8 | p[i];
    if (n > size_ - 8) throw std::runtime_error(path + ": the header is cut off");
    const char* h = reinterpret_cast<const char*>(p + 8);
    const Json head = Json::parse(h, h + n);
    const uint8_t* data = p + 8 + n;
    const uint64_t avail = size_ - 8 - n;
    for (const auto& kv : head.members()) {
      if (kv.first == "__metadata__") continue;
      Tensor t;
      t.dtype = kv.second.at("dtype").string();
      for (const Json& d : kv.second.at("shape").items()) t.shape.push_back(d.integer());
      const auto& off = kv.second.at("data_offsets").items();
      const long width = t.dtype == "BF16" || t.dtype == "F16" ? 2 : t.dtype == "F32" || t.dtype == "I32" ? 4 : 0;
      if (off.size() != 2 || width == 0)
        throw std::runtime_error("tensor '" + kv.first + "': unsupported dtype " + t.dtype);
      const uint64_t a = (uint64_t)off[0].integer(), b = (uint64_t)off[1].integer();
      if (a > b || b > avail || (long)(b - a) != t.count() * width)
        throw std::runtime_error("tensor '" + kv.first + "': bad data_offsets");
      t.data = data + a;
      tensors_[kv.first] = t;
    }
  }
  void* map_ = nullptr;
  size_t size_ = 0;
  std::map<std::string, Tensor> tensors_;
};

}  // namespace hip
}  // namespace lightseq
