// safetensors.hpp -- reader of a safetensors file: u64 header length, a JSON header {name: {dtype, shape, data_offsets}}, the data.
// The file is mapped; a tensor's bytes go from the mapping to the device as GGUF's do (gguf.hpp).
#pragma once
#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <map>

#include "hip_tensor.hpp"
#include "json.hpp"

namespace crabml_host {

struct SafeTensorInfo {
  std::string dtype;
  std::vector<size_t> shape;
  const uint8_t* data = nullptr;
  size_t len = 0;
  size_t elems() const {
    size_t n = 1;
    for (size_t d : shape) n *= d;
    return n;
  }
};

class SafeTensorsFile {
 public:
  explicit SafeTensorsFile(const std::string& path) {
    fd_ = ::open(path.c_str(), O_RDONLY | O_CLOEXEC);
    struct stat st;
    if (fd_ < 0 || ::fstat(fd_, &st) != 0) throw_io("cannot open " + path);
    len_ = (size_t)st.st_size;
    if (len_ < 8) throw_format(path + " is too short");
    void* m = ::mmap(nullptr, len_, PROT_READ, MAP_PRIVATE, fd_, 0);
    if (m == MAP_FAILED) throw_io("cannot map " + path);
    base_ = (const uint8_t*)m;
    uint64_t n = 0;
    for (int i = 7; i >= 0; i--) n = n << 8 | base_[i];
    if (n > len_ - 8) throw_format(path + ": the header is longer than the file");
    const uint8_t* data = base_ + 8 + n;
    const size_t data_len = len_ - 8 - (size_t)n;
    try {
      const Json head = Json::parse((const char*)base_ + 8, (size_t)n);
      for (const auto& f : head.fields()) {
        if (f.first == "__metadata__") continue;
        SafeTensorInfo t;
        t.dtype = f.second.at("dtype").str();
        for (const Json& d : f.second.at("shape").items()) t.shape.push_back(d.size());
        const auto& o = f.second.at("data_offsets").items();
        if (o.size() != 2 || o[0].size() > o[1].size() || o[1].size() > data_len) throw Error(ErrorKind::FormatError, "tensor " + f.first + " lies outside the data");
        size_t n_el = 1;
        for (size_t d : t.shape)
          if (__builtin_mul_overflow(n_el, d, &n_el)) throw Error(ErrorKind::FormatError, "tensor " + f.first + ": element count overflows");
        t.data = data + o[0].size();
        t.len = o[1].size() - o[0].size();
        tensors_[f.first] = std::move(t);
      }
    } catch (...) {
      release();
      throw;
    }
  }
  ~SafeTensorsFile() { release(); }
  SafeTensorsFile(const SafeTensorsFile&) = delete;
  SafeTensorsFile& operator=(const SafeTensorsFile&) = delete;

  const std::map<std::string, SafeTensorInfo>& tensors() const { return tensors_; }
  bool has(const std::string& name) const { return tensors_.count(name) != 0; }

  // the tensor on the device, its shape checked ({} = a single number)
  HipTensor load(const std::string& name, const std::vector<size_t>& shape, const HipTensorDeviceRef& device) const {
    auto it = tensors_.find(name);
    if (it == tensors_.end()) throw Error(ErrorKind::TensorNotFound, "failed to find tensor " + name);
    const SafeTensorInfo& t = it->second;
    if (t.shape != shape) throw Error(ErrorKind::ModelError, "tensor " + name + " is " + fmt_dims(t.shape) + ", the configuration wants " + fmt_dims(shape));
    GGMLType type;
    if (t.dtype == "BF16")
      type = GGMLType::BF16;
    else if (t.dtype == "F32")
      type = GGMLType::F32;
    else if (t.dtype == "F16")
      type = GGMLType::F16;
    else
      throw Error(ErrorKind::NotImplemented, "tensor " + name + ": dtype " + t.dtype + " is not supported by the hip backend");
    const size_t bytes = t.elems() * (type == GGMLType::F32 ? 4 : 2);
    if (bytes != t.len) throw Error(ErrorKind::FormatError, "tensor " + name + " holds " + std::to_string(t.len) + " bytes, its shape wants " + std::to_string(bytes));
    return HipTensor::from_cpu(t.data, bytes, shape.empty() ? std::vector<size_t>{1} : shape, type, device);
  }

 private:
  void release() {
    if (base_) ::munmap((void*)base_, len_);
    if (fd_ >= 0) ::close(fd_);
    base_ = nullptr;
    fd_ = -1;
  }
  [[noreturn]] void throw_io(const std::string& m) {
    release();
    throw Error(ErrorKind::IOError, m);
  }
  [[noreturn]] void throw_format(const std::string& m) {
    release();
    throw Error(ErrorKind::FormatError, m);
  }
  int fd_ = -1;
  const uint8_t* base_ = nullptr;
  size_t len_ = 0;
  std::map<std::string, SafeTensorInfo> tensors_;
};

}  // namespace crabml_host
