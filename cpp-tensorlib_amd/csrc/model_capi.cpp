// C entry points over the model registry (include/tl/models.h): open a model by its path, feed it
// tokens, generate. Part of libtl_qwen.so.
#include <cstdint>
#include <cstring>
#include <memory>
#include <string>

#include "../include/tl/models.h"

using namespace tl;

namespace {
thread_local std::string g_error;
struct handle {
  std::unique_ptr<models::any> p;
  models::of<lusadra::model>* lus = nullptr;   // the same object, where it is one
  loops::captured_step<lusadra::model> cap;
};
template <class F>
void* guarded(F f) {
  g_error.clear();
  try {
    return f();
  } catch (const std::exception& e) {
    g_error = e.what();
    return nullptr;
  }
}
}  // namespace

extern "C" {

const char* tlm_error() { return g_error.c_str(); }

// exact != 0: prompt products exact in f32; q4 != 0: int4 weights (GGUF only). NULL on error.
void* tlm_open(const char* path, int64_t max_ctx, int64_t chunk, int exact, int q4) {
  return guarded([&]() -> void* {
    models::options o;
    o.max_ctx = max_ctx;
    o.chunk = chunk;
    o.exact = exact != 0;
    o.q4 = q4 != 0;
    auto h = std::make_unique<handle>();
    h->p = models::open(path, o);
    h->lus = dynamic_cast<models::of<lusadra::model>*>(h->p.get());
    return h.release();
  });
}
// A Lusadra model of the given configuration (JSON text) with seeded weights, for throughput runs.
void* tlm_random_lusadra(const char* config, uint32_t seed, int64_t rank, int64_t max_ctx, int64_t chunk, int exact) {
  return guarded([&]() -> void* {
    auto h = std::make_unique<handle>();
    auto p = std::make_unique<models::of<lusadra::model>>(lusadra::kArchitecture, chunk);
    p->m.exact = exact != 0;
    lusadra::load_random(p->m, json::parse(config), seed, rank, max_ctx, chunk);
    h->lus = p.get();
    h->p = std::move(p);
    return h.release();
  });
}
void tlm_close(void* hv) {
  auto* h = static_cast<handle*>(hv);
  h->cap.destroy();
  delete h;
}
const char* tlm_architecture(void* hv) { return static_cast<handle*>(hv)->p->architecture(); }
int64_t tlm_vocab(void* hv) { return static_cast<handle*>(hv)->p->vocab(); }
int64_t tlm_capacity(void* hv) { return static_cast<handle*>(hv)->p->capacity(); }
int64_t tlm_pos(void* hv) { return static_cast<handle*>(hv)->p->pos(); }
void tlm_reset(void* hv) { static_cast<handle*>(hv)->p->reset(); }
// The next n tokens of the sequence; out: [n_want, vocab] logits of the places listed in want.
int tlm_feed(void* hv, const int64_t* tokens, int64_t n, const int64_t* want, int64_t n_want, float* out) {
  return static_cast<handle*>(hv)->p->feed(tokens, n, want, n_want, out) ? 0 : -1;
}
int64_t tlm_generate(void* hv, int64_t next, int64_t n, int32_t* out) {
  return static_cast<handle*>(hv)->p->generate(next, n, out);
}

// ---- Lusadra: launch forms, diagnostics, throughput ------------------------------------------------
int tlm_set_fused(void* hv, int on) {
  auto* h = static_cast<handle*>(hv);
  if (!h->lus) return -1;
  h->lus->m.fused = on != 0;
  return 0;
}
// Residual stream after every layer run of one chunk at the current position: out [runs][n][width].
int64_t tlm_layer_runs(void* hv) {
  auto* h = static_cast<handle*>(hv);
  return h->lus ? (int64_t)h->lus->m.runs.size() : -1;
}
int tlm_trace_chunk(void* hv, const int64_t* tokens, int64_t n, float* out) {
  auto* h = static_cast<handle*>(hv);
  if (!h->lus) return -1;
  auto& M = h->lus->m;
  if (M.pos + n > M.max_ctx || !lusadra::stage_chunk(M, tokens, n) || !lusadra::chunk_layers(M, n, out)) return -1;
  M.pos += n;
  return 0;
}
// One step at a fixed position, recorded and replayed; one eager step; chunks queued with no sync.
int tlm_capture_step(void* hv, int64_t token, int64_t pos) {
  auto* h = static_cast<handle*>(hv);
  if (!h->lus) return -1;
  h->cap.destroy();
  return lusadra::stage_embed(h->lus->m, token) && h->cap.capture(h->lus->m, pos) ? 0 : -1;
}
int tlm_replay_step(void* hv) { return static_cast<handle*>(hv)->cap.replay() ? 0 : -1; }
int tlm_eager_step(void* hv, int64_t token, int64_t pos) {
  auto* h = static_cast<handle*>(hv);
  return h->lus && lusadra::stage_embed(h->lus->m, token) && lusadra::step_layers(h->lus->m, pos) ? 0 : -1;
}
int tlm_stage_chunk(void* hv, const int64_t* tokens, int64_t n) {
  auto* h = static_cast<handle*>(hv);
  return h->lus && lusadra::stage_chunk(h->lus->m, tokens, n) ? 0 : -1;
}
int tlm_chunk_layers(void* hv, int64_t n, int64_t pos0) {
  auto* h = static_cast<handle*>(hv);
  if (!h->lus || pos0 + n > h->lus->m.max_ctx) return -1;
  h->lus->m.pos = pos0;
  return lusadra::chunk_layers(h->lus->m, n) ? 0 : -1;
}

}  // extern "C"
