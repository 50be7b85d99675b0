#pragma once

// The models this build knows, behind one interface: a path is opened by what it holds - a GGUF file by
// its general.architecture, a folder by the "architecture" of its config.json - and the result takes
// tokens in portions of any size and generates greedily (loops::sequence).

#include <sys/stat.h>

#include <fstream>
#include <memory>
#include <sstream>
#include <stdexcept>
#include <string>

#include "decode_loop.h"
#include "gguf.h"
#include "json.h"
#include "lusadra.h"
#include "qwen_decode.h"

namespace tl {
namespace models {

struct options {
  int64_t max_ctx = 4096;
  int64_t chunk = 512;         // longest prompt chunk
  bool exact = false;          // prompt products exact in f32, not in two rounded terms per operand
  bool q4 = false;             // int4 weights (models loaded from GGUF)
};

class any {
 public:
  virtual ~any() = default;
  virtual const char* architecture() const = 0;
  virtual int64_t vocab() const = 0;
  virtual int64_t capacity() const = 0;
  virtual int64_t pos() const = 0;
  virtual void reset() = 0;
  virtual bool feed(const int64_t* tokens, int64_t n, const int64_t* want, int64_t n_want, float* out) = 0;
  virtual int64_t generate(int64_t next, int64_t n, int32_t* out) = 0;
};

template <class M>
class of : public any {
  std::string name_;
  int64_t chunk_;

 public:
  M m;
  loops::sequence<M> seq{m};
  of(std::string name, int64_t chunk) : name_(std::move(name)), chunk_(chunk) {}
  const char* architecture() const override { return name_.c_str(); }
  int64_t vocab() const override { return vocab_size(m); }
  int64_t capacity() const override { return context_capacity(m); }
  int64_t pos() const override { return seq.pos(); }
  void reset() override { seq.reset(); }
  bool feed(const int64_t* tokens, int64_t n, const int64_t* want, int64_t n_want, float* out) override {
    return seq.feed(tokens, n, want, n_want, out, chunk_);
  }
  int64_t generate(int64_t next, int64_t n, int32_t* out) override { return seq.generate(next, n, out); }
};

// ---- folders: config.json + model.safetensors ---------------------------------------------------
inline std::unique_ptr<any> open_lusadra(const json::value& cfg, const std::string& dir, const options& o) {
  auto p = std::make_unique<of<lusadra::model>>(lusadra::kArchitecture, o.chunk);
  p->m.exact = o.exact;
  lusadra::load(p->m, cfg, dir, o.max_ctx, o.chunk);
  return p;
}

struct entry {
  const char* architecture;
  std::unique_ptr<any> (*open)(const json::value&, const std::string&, const options&);
};
constexpr entry kFolders[] = {{lusadra::kArchitecture, open_lusadra}};

// ---- GGUF files ---------------------------------------------------------------------------------
inline std::unique_ptr<any> open_gguf(const std::string& path, const options& o) {
  const gguf::model g(path);
  auto p = std::make_unique<of<qwen::model>>("qwen2", o.chunk);
  p->m.prompt_f16 = !o.exact;
  std::string why;
  if (!qwen::load_gguf(p->m, g, o.q4 ? qwen::wfmt::q4 : qwen::wfmt::bf16_row, o.max_ctx, &why)) throw std::runtime_error(why);
  return p;
}

inline json::value read_config(const std::string& dir) {
  std::ifstream in(dir + "/config.json", std::ios::binary);
  if (!in) throw std::runtime_error(dir + "/config.json: cannot open");
  std::stringstream text;
  text << in.rdbuf();
  return json::parse(text.str());
}

// Throws std::runtime_error with the reason.
inline std::unique_ptr<any> open(const std::string& path, const options& o) {
  struct stat st;
  if (::stat(path.c_str(), &st) != 0) throw std::runtime_error(path + ": not found");
  if (!S_ISDIR(st.st_mode)) return open_gguf(path, o);
  const json::value cfg = read_config(path);
  const std::string& arch = cfg.at("architecture").str();
  for (const entry& e : kFolders)
    if (arch == e.architecture) return e.open(cfg, path, o);
  throw std::runtime_error(path + ": unknown architecture " + arch);
}

}  // namespace models
}  // namespace tl
