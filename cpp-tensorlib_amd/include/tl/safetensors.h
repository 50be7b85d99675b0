#pragma once

// safetensors files: an 8-byte little-endian header length, that many bytes of JSON
// (name -> dtype, shape, data_offsets), then the tensors' bytes. The file is mapped, tensors point into
// the mapping; every offset and size is checked against the file before use.

#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <cstdint>
#include <map>
#include <stdexcept>
#include <string>
#include <vector>

#include "json.h"

namespace tl {
namespace safetensors {

struct tensor {
  std::string dtype;             // "BF16", "F32", ...
  std::vector<int64_t> shape;    // empty: one number
  const void* data = nullptr;
  int64_t bytes = 0;
  int64_t elements() const {
    int64_t n = 1;
    for (int64_t d : shape) n *= d;
    return n;
  }
};

inline int64_t dtype_bytes(const std::string& t) {
  if (t == "F64" || t == "I64" || t == "U64") return 8;
  if (t == "F32" || t == "I32" || t == "U32") return 4;
  if (t == "F16" || t == "BF16" || t == "I16" || t == "U16") return 2;
  if (t == "I8" || t == "U8" || t == "BOOL") return 1;
  return 0;
}

class file {
  void* map_ = MAP_FAILED;
  size_t size_ = 0;
  std::map<std::string, tensor> tensors_;

  void parse(const std::string& path) {
    const auto bad = [&](const std::string& what) { throw std::runtime_error(path + ": " + what); };
    if (size_ < 8) bad("too short");
    const unsigned char* p = static_cast<const unsigned char*>(map_);
    uint64_t hn = 0;
    for (int i = 7; i >= 0; i--) hn = hn << 8 | p[i];
    if (hn > size_ - 8) bad("header longer than the file");
    const json::value h = json::parse(reinterpret_cast<const char*>(p) + 8, static_cast<size_t>(hn));
    const uint64_t room = size_ - 8 - hn;
    for (const auto& e : h.o) {
      if (e.first == "__metadata__") continue;
      tensor t;
      t.dtype = e.second.at("dtype").str();
      int64_t n = 1;
      for (const auto& d : e.second.at("shape").items()) {
        const int64_t v = d.integer();
        if (v < 0 || (v > 0 && n > (int64_t(1) << 50) / v)) bad(e.first + ": bad shape");
        t.shape.push_back(v);
        n *= v;
      }
      const auto& off = e.second.at("data_offsets").items();
      const int64_t es = dtype_bytes(t.dtype);
      if (off.size() != 2 || es == 0) bad(e.first + ": bad entry");
      const int64_t b = off[0].integer(), f = off[1].integer();
      if (b < 0 || f < b || static_cast<uint64_t>(f) > room || f - b != n * es) bad(e.first + ": bad offsets");
      t.data = p + 8 + hn + b;
      t.bytes = f - b;
      tensors_.emplace(e.first, std::move(t));
    }
  }

 public:
  explicit file(const std::string& path) {
    const int fd = ::open(path.c_str(), O_RDONLY | O_CLOEXEC);
    if (fd < 0) throw std::runtime_error(path + ": cannot open");
    struct stat st;
    if (::fstat(fd, &st) == 0 && st.st_size > 0) {
      size_ = static_cast<size_t>(st.st_size);
      map_ = ::mmap(nullptr, size_, PROT_READ, MAP_PRIVATE, fd, 0);
    }
    ::close(fd);
    if (map_ == MAP_FAILED) throw std::runtime_error(path + ": cannot map");
    try {
      parse(path);
    } catch (...) {
      ::munmap(map_, size_);
      throw;
    }
  }
  file(const file&) = delete;
  file& operator=(const file&) = delete;
  ~file() {
    if (map_ != MAP_FAILED) ::munmap(map_, size_);
  }
  const tensor* find(const std::string& name) const {
    auto it = tensors_.find(name);
    return it == tensors_.end() ? nullptr : &it->second;
  }
  const std::map<std::string, tensor>& tensors() const { return tensors_; }
};

}  // namespace safetensors
}  // namespace tl
