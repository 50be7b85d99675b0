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
using handle = models::any;
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
    return models::open(path, o).release();
  });
}
// A model of the given configuration (JSON text) with seeded weights, for throughput runs. rank: of Lusadra's
// decay inputs.
void* tlm_random(const char* config, uint32_t seed, int64_t rank, int64_t max_ctx, int64_t chunk, int exact) {
  return guarded([&]() -> void* {
    models::options o;
    o.max_ctx = max_ctx;
    o.chunk = chunk;
    o.exact = exact != 0;
    return models::random(config, seed, rank, o).release();
  });
}
void tlm_close(void* hv) { delete static_cast<handle*>(hv); }
const char* tlm_architecture(void* hv) { return static_cast<handle*>(hv)->architecture(); }
int64_t tlm_vocab(void* hv) { return static_cast<handle*>(hv)->vocab(); }
int64_t tlm_capacity(void* hv) { return static_cast<handle*>(hv)->capacity(); }
int64_t tlm_pos(void* hv) { return static_cast<handle*>(hv)->pos(); }
void tlm_reset(void* hv) { static_cast<handle*>(hv)->reset(); }
// The next n tokens of the sequence; out: [n_want, vocab] logits of the places listed in want.
int tlm_feed(void* hv, const int64_t* tokens, int64_t n, const int64_t* want, int64_t n_want, float* out) {
  return static_cast<handle*>(hv)->feed(tokens, n, want, n_want, out) ? 0 : -1;
}
int64_t tlm_generate(void* hv, int64_t next, int64_t n, int32_t* out) { return static_cast<handle*>(hv)->generate(next, n, out); }

// ---- launch forms, diagnostics, throughput (designs read from folders) ------------------------------
int tlm_set_fused(void* hv, int on) { return static_cast<handle*>(hv)->set_fused(on != 0) ? 0 : -1; }
// Residual stream after every layer run of one chunk at the current position: out [runs][n][width].
int64_t tlm_layer_runs(void* hv) { return static_cast<handle*>(hv)->runs(); }
int tlm_trace_chunk(void* hv, const int64_t* tokens, int64_t n, float* out) { return static_cast<handle*>(hv)->trace(tokens, n, out) ? 0 : -1; }
// One step at a fixed position, recorded and replayed; one eager step; chunks queued with no sync.
int tlm_capture_step(void* hv, int64_t token, int64_t pos) { return static_cast<handle*>(hv)->record_step(token, pos) ? 0 : -1; }
int tlm_replay_step(void* hv) { return static_cast<handle*>(hv)->replay_recorded() ? 0 : -1; }
int tlm_eager_step(void* hv, int64_t token, int64_t pos) { return static_cast<handle*>(hv)->eager_step(token, pos) ? 0 : -1; }
int tlm_stage_chunk(void* hv, const int64_t* tokens, int64_t n) { return static_cast<handle*>(hv)->queue_tokens(tokens, n) ? 0 : -1; }
int tlm_chunk_layers(void* hv, int64_t n, int64_t pos0) { return static_cast<handle*>(hv)->queue_chunk(n, pos0) ? 0 : -1; }

}  // extern "C"
