#pragma once

// Where a model's tensors come from: a safetensors file, or a generator for throughput runs. Shared by the
// designs that are read from folders.

#include <cmath>
#include <cstdint>
#include <cstring>
#include <stdexcept>
#include <string>
#include <vector>

#include "safetensors.h"
#include "types.h"

namespace tl {
namespace source {

inline int64_t up(int64_t n, int64_t to) { return (n + to - 1) / to * to; }

// Where tensors come from: a file, or a generator for throughput runs. Values are bf16 bits.
struct reader {
  virtual ~reader() = default;
  // rows x cols of `name` (checked against the shape; cols 0: a vector, rows 0: one number)
  virtual void read(const std::string& name, int64_t rows, int64_t cols, uint16_t* dst, int64_t ld) = 0;
  virtual int64_t rows_of(const std::string& name) = 0;
};

struct file : reader {
  const safetensors::file& f;
  explicit file(const safetensors::file& st) : f(st) {}
  const safetensors::tensor& get(const std::string& name) const {
    const safetensors::tensor* t = f.find(name);
    if (!t) throw std::runtime_error("missing tensor " + name);
    if (t->dtype != "BF16") throw std::runtime_error(name + ": bf16 expected");
    return *t;
  }
  void read(const std::string& name, int64_t rows, int64_t cols, uint16_t* dst, int64_t ld) override {
    const safetensors::tensor& t = get(name);
    std::vector<int64_t> want;
    if (rows) want.push_back(rows);
    if (cols) want.push_back(cols);
    // a single number may be stored with or without a dimension of 1
    const bool one = !rows && !cols && t.elements() == 1;
    if (!one && t.shape != want) throw std::runtime_error(name + ": shape does not match the configuration");
    const int64_t r = rows ? rows : 1, n = cols ? cols : 1;
    const char* p = static_cast<const char*>(t.data);
    if (!cols) {                       // a vector: contiguous
      std::memcpy(dst, p, (size_t)r * 2);
      return;
    }
    for (int64_t i = 0; i < r; i++) std::memcpy(dst + i * ld, p + i * n * 2, (size_t)n * 2);
  }
  int64_t rows_of(const std::string& name) override {
    const safetensors::tensor& t = get(name);
    if (t.shape.empty()) throw std::runtime_error(name + ": a matrix expected");
    return t.shape[0];
  }
};

// Seeded values of a size that keeps activations finite; for throughput runs.
struct random : reader {
  int64_t rank;
  std::vector<float> block;            // uniform in [-1, 1), drawn once and walked through again and again
  size_t at = 0;
  random(uint32_t seed, int64_t low_rank) : rank(low_rank), block((size_t)(1 << 20) + 7) {
    uint32_t s = seed * 2654435761u + 1u;
    for (auto& v : block) {
      s ^= s << 13; s ^= s >> 17; s ^= s << 5;
      v = (float)(int32_t)s * (1.0f / 2147483648.0f);
    }
  }
  void read(const std::string&, int64_t rows, int64_t cols, uint16_t* dst, int64_t ld) override {
    const int64_t r = rows ? rows : 1, n = cols ? cols : 1;
    const float amp = cols ? std::sqrt(3.0f / (float)n) : 1.0f;
    for (int64_t i = 0; i < r; i++)
      for (int64_t k = 0; k < n; k++) {
        dst[i * (cols ? ld : 1) + k] = f32_to_bf16(amp * block[at]);
        if (++at == block.size()) at = 0;
      }
  }
  int64_t rows_of(const std::string&) override { return rank; }
};

struct part { std::string name; int64_t rows, at; };   // rows of a stacked matrix

}  // namespace source

}  // namespace tl
