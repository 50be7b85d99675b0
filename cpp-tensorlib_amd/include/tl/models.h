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
#include "girirax.h"
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

// Models that offer what measuring and checking layer by layer needs: launch forms, the residual stream
// after every layer, single steps and chunks without the loops.
template <class M>
struct inspectable { static constexpr bool value = false; };
template <>
struct inspectable<lusadra::model> { static constexpr bool value = true; };
template <>
struct inspectable<girirax::model> { static constexpr bool value = true; };

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
  // inspectable models; false (-1) elsewhere
  virtual bool set_fused(bool on) = 0;
  virtual int64_t runs() const = 0;
  virtual bool trace(const int64_t* tokens, int64_t n, float* out) = 0;   // [runs][n][width] at the current position
  virtual bool record_step(int64_t token, int64_t pos) = 0;                    // recorded at a fixed position, and replayed
  virtual bool replay_recorded() = 0;
  virtual bool eager_step(int64_t token, int64_t pos) = 0;
  virtual bool queue_tokens(const int64_t* tokens, int64_t n) = 0;               // then queue_chunk, with no sync
  virtual bool queue_chunk(int64_t n, int64_t pos0) = 0;
};

template <class M>
class of : public any {
  std::string name_;
  int64_t chunk_;

 public:
  M m;
  loops::sequence<M> seq{m};
  loops::captured_step<M> step;
  of(std::string name, int64_t chunk) : name_(std::move(name)), chunk_(chunk) {}
  ~of() override { step.destroy(); }
  const char* architecture() const override { return name_.c_str(); }
  int64_t vocab() const override { return vocab_size(m); }
  int64_t capacity() const override { return context_capacity(m); }
  int64_t pos() const override { return seq.pos(); }
  void reset() override { seq.reset(); }
  bool feed(const int64_t* tokens, int64_t n, const int64_t* want, int64_t n_want, float* out) override {
    return seq.feed(tokens, n, want, n_want, out, chunk_);
  }
  int64_t generate(int64_t next, int64_t n, int32_t* out) override { return seq.generate(next, n, out); }

  bool set_fused(bool on) override {
    if constexpr (inspectable<M>::value) m.fused = on;
    return inspectable<M>::value;
  }
  int64_t runs() const override {
    if constexpr (inspectable<M>::value) return layer_runs(m);
    return -1;
  }
  bool trace(const int64_t* tokens, int64_t n, float* out) override {
    if constexpr (inspectable<M>::value) {
      const int64_t p = seq.pos();
      if (p + n > capacity() || !stage_chunk(m, tokens, n) || !chunk_layers(m, n, out)) return false;
      set_cache_pos(m, p + n);
      return true;
    }
    return false;
  }
  bool record_step(int64_t token, int64_t pos) override {
    if constexpr (inspectable<M>::value) {
      step.destroy();
      return stage_embed(m, token) && step.capture(m, pos);
    }
    return false;
  }
  bool replay_recorded() override { return step.replay(); }
  bool eager_step(int64_t token, int64_t pos) override {
    if constexpr (inspectable<M>::value) return stage_embed(m, token) && step_layers(m, pos);
    return false;
  }
  bool queue_tokens(const int64_t* tokens, int64_t n) override {
    if constexpr (inspectable<M>::value) return stage_chunk(m, tokens, n);
    return false;
  }
  bool queue_chunk(int64_t n, int64_t pos0) override {
    if constexpr (inspectable<M>::value) {
      if (pos0 + n > capacity()) return false;
      set_cache_pos(m, pos0);
      return chunk_layers(m, n, nullptr);
    }
    return false;
  }
};

// ---- folders: config.json + model.safetensors ---------------------------------------------------
inline std::unique_ptr<any> open_lusadra(const json::value& cfg, const std::string& dir, const options& o) {
  auto p = std::make_unique<of<lusadra::model>>(lusadra::kArchitecture, o.chunk);
  p->m.exact = o.exact;
  lusadra::load(p->m, cfg, dir, o.max_ctx, o.chunk);
  return p;
}

inline std::unique_ptr<any> open_girirax(const json::value& cfg, const std::string& dir, const options& o) {
  auto p = std::make_unique<of<girirax::model>>(girirax::kArchitecture, o.chunk);
  p->m.exact = o.exact;
  girirax::load(p->m, cfg, dir, o.max_ctx, o.chunk);
  return p;
}
// The same designs with seeded weights; rank: of Lusadra's decay inputs, which its configuration does not give.
inline std::unique_ptr<any> random_lusadra(const json::value& cfg, uint32_t seed, int64_t rank, const options& o) {
  auto p = std::make_unique<of<lusadra::model>>(lusadra::kArchitecture, o.chunk);
  p->m.exact = o.exact;
  lusadra::load_random(p->m, cfg, seed, rank, o.max_ctx, o.chunk);
  return p;
}
inline std::unique_ptr<any> random_girirax(const json::value& cfg, uint32_t seed, int64_t, const options& o) {
  auto p = std::make_unique<of<girirax::model>>(girirax::kArchitecture, o.chunk);
  p->m.exact = o.exact;
  girirax::load_random(p->m, cfg, seed, o.max_ctx, o.chunk);
  return p;
}

struct entry {
  const char* architecture;
  std::unique_ptr<any> (*open)(const json::value&, const std::string&, const options&);
  std::unique_ptr<any> (*random)(const json::value&, uint32_t seed, int64_t rank, const options&);
};
constexpr entry kFolders[] = {{lusadra::kArchitecture, open_lusadra, random_lusadra},
                              {girirax::kArchitecture, open_girirax, random_girirax}};
inline const entry& folder_entry(const json::value& cfg, const std::string& where) {
  const std::string& arch = cfg.at("architecture").str();
  for (const entry& e : kFolders)
    if (arch == e.architecture) return e;
  throw std::runtime_error(where + ": unknown architecture " + arch);
}

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
  return folder_entry(cfg, path).open(cfg, path, o);
}
// A model of a configuration (the text of a config.json) with seeded weights, for throughput runs.
inline std::unique_ptr<any> random(const std::string& config, uint32_t seed, int64_t rank, const options& o) {
  const json::value cfg = json::parse(config);
  return folder_entry(cfg, "config").random(cfg, seed, rank, o);
}

}  // namespace models
}  // namespace tl
