#pragma once

// Decoding loops over any model that offers the small set of functions named below (found by
// argument-dependent lookup): a prompt in chunks, one eager step, a step recorded at a fixed position,
// a decoder that replays one recorded graph with the position on the device (the counterpart of
// bench/cuda/qwen_model.h:791-905), a greedy loop whose tokens never leave the device, and `sequence`,
// which feeds tokens to a model in whatever portions they come.
//
//   int64_t vocab_size(const M&), context_capacity(const M&), cache_pos(const M&), longest_chunk(const M&)
//   void set_cache_pos(M&, int64_t)                 what the caches hold counts up to this position
//   bool stage_embed(M&, token)                     input of the next step from the host
//   bool step_layers(M&, pos, d_pos, advance)       one token -> logits_device(M); no sync, capturable;
//                                                   with d_pos (a device scalar) the launches do not
//                                                   depend on the position, and advance moves it on
//   bool step_layers_from(M&, d_tok, d_pos)         the same, token id on the device, not advanced
//   bool reserve_device_steps(M&, device_tokens)    allocations of the two; false: not offered
//   bool prompt_chunk(M&, tokens, T)                T tokens at cache_pos; normed rows in chunk_rows(M)
//   void* chunk_rows(M&), logits_device(M&); int64_t chunk_row_width(const M&)
//   const float* logits_host(const M&); const weights::linear& head(const M&)
//
// A step at a position must be repeatable at that position: recording runs it once before.

#include <algorithm>
#include <cstdint>
#include <vector>

#include "hip.h"
#include "linear.h"

namespace tl {
namespace loops {

// embed -> layers -> device argmax. Returns the greedy token, or -1 when any
// launch was declined.
template <class M>
int64_t step_greedy(M& m, int64_t token, int64_t pos) {
  if (!stage_embed(m, token) || !step_layers(m, pos)) return -1;
  int64_t idx = -1;
  if (!hip::argmax(logits_device(m), vocab_size(m), &idx)) return -1;
  return idx;
}

// Host view of the logits the last step left on the device.
template <class M>
const float* logits(M& m) {
  hip::sync_to_host(logits_device(m), false);
  return logits_host(m);
}

// Consume a prompt in chunks; logits of its LAST token land in logits_device (only
// that row is ever read, so only it meets the lm_head: qm:396-401).
template <class M>
bool prefill(M& m, const int64_t* tokens, int64_t n, int64_t chunk = 512) {
  if (n <= 0 || chunk <= 0) return false;
  if (longest_chunk(m) > 0) chunk = std::min(chunk, longest_chunk(m));
  bool ok = true;
  int64_t last_T = 0;
  for (int64_t t0 = 0; t0 < n && ok; t0 += chunk) {
    last_T = std::min(chunk, n - t0);
    ok = prompt_chunk(m, tokens + t0, last_T);
  }
  if (!ok) return false;
  void* last = static_cast<char*>(chunk_rows(m)) + (last_T - 1) * chunk_row_width(m) * 4;
  return gemv(head(m), last, logits_device(m));
}

// One decode step recorded as a hipGraph at a FIXED position (the throughput
// measurement replays the same step; replaying re-writes the same cache row).
template <class M>
struct captured_step {
  void* graph = nullptr;
  bool capture(M& m, int64_t pos) {
    // warm: lets the library size its scratch before the capture opens
    if (!step_layers(m, pos)) return false;
    hip::flush();
    if (!hip::capture_begin()) return false;
    const bool ok = step_layers(m, pos);
    graph = hip::capture_end();
    return ok && graph != nullptr;
  }
  bool replay() { return hip::graph_launch(graph); }
  void destroy() {
    hip::graph_destroy(graph);
    graph = nullptr;
  }
};

// Greedy decoding with the whole token loop on the device: one recorded graph does
//   embedding gather of *d_tok -> layers at *d_pos -> lm_head -> argmax -> *d_tok,
//   history[*d_pos] = *d_tok, *d_pos += 1
// so consecutive tokens are queued back to back with no host round trip between them
// (the reference stages each embedding on the host and reads every argmax back:
// qm:530-535, 642-647). The host reads the generated ids from the history afterwards.
template <class M>
struct greedy_loop {
  void *d_pos = nullptr, *d_tok = nullptr, *history = nullptr, *graph = nullptr;
  float* history_host = nullptr;
  int64_t cur_pos = 0, max_ctx = 0;

  bool init(M& m, int64_t first_id, int64_t pos) {
    if (first_id < 0 || first_id >= vocab_size(m)) return false;   // later ids are argmax results, in range by construction
    max_ctx = context_capacity(m);
    cur_pos = pos;
    if (!reserve_device_steps(m, true)) return false;
    d_pos = hip::alloc(4, nullptr);
    d_tok = hip::alloc(4, nullptr);
    history = hip::alloc(max_ctx * 4, &history_host);
    if (!d_pos || !d_tok || !history) return false;
    auto one = [&]() {
      bool ok = step_layers_from(m, d_tok, d_pos);
      ok = ok && hip::argmax_async(logits_device(m), vocab_size(m), d_tok);
      return ok && hip::token_advance(d_pos, d_tok, history, max_ctx);
    };
    hip::upload_u32(d_pos, (unsigned)pos);
    hip::upload_u32(d_tok, (unsigned)first_id);
    if (!one()) return false;            // warm run (sizes the library's scratch)
    hip::flush();
    hip::upload_u32(d_pos, (unsigned)pos);
    hip::upload_u32(d_tok, (unsigned)first_id);
    if (!hip::capture_begin()) return false;
    const bool ok = one();
    graph = hip::capture_end();
    if (!ok && graph) { hip::graph_destroy(graph); graph = nullptr; }
    return graph != nullptr;
  }
  // Queue n greedy steps (no sync). Returns how many were queued before the cache filled.
  int64_t run(int64_t n) {
    int64_t done = 0;
    while (done < n && cur_pos < max_ctx && graph && hip::graph_launch(graph)) {
      cur_pos++;
      done++;
    }
    return done;
  }
  // The token generated at position p (p in [first pos, cur_pos)); blocks until the queue drained.
  const int32_t* tokens() {
    hip::sync_to_host(history, false);
    return reinterpret_cast<const int32_t*>(history_host);
  }
  void sync_host_pos(M& m) const { set_cache_pos(m, cur_pos); }
  void destroy() {
    if (graph) hip::graph_destroy(graph);
    for (void* b : {d_pos, d_tok, history})
      if (b) hip::release(b, 0, nullptr);
    graph = d_pos = d_tok = history = nullptr;
  }
};

// A decode loop on ONE recorded graph (qm:791-905): the position lives in a device
// scalar that the recorded forward advances itself, so feed()/step() replay the same
// graph for every token. Falls back to the imperative path when capture is not
// available; callers never branch on ok().
template <class M>
struct captured_decoder {
  void* d_pos = nullptr;
  void* graph = nullptr;
  int64_t cur_pos = 0, max_ctx = 0;

  // Record the forward at `pos` (the first position this decoder will process).
  bool init(M& m, int64_t first_id, int64_t pos) {
    max_ctx = context_capacity(m);
    cur_pos = pos;
    if (!reserve_device_steps(m, false)) return false;
    d_pos = hip::alloc(4, nullptr);
    if (!d_pos) return false;
    if (!stage_embed(m, first_id)) return false;
    hip::upload_u32(d_pos, (unsigned)pos);
    // warm run: real launches (they also size the library's scratch); it advances d_pos
    // and writes cache row pos, which the first recorded step rewrites identically
    if (!step_layers(m, pos, d_pos)) return false;
    hip::flush();
    hip::upload_u32(d_pos, (unsigned)pos);
    if (!hip::capture_begin()) return false;
    const bool ok = step_layers(m, pos, d_pos);  // recorded, not executed
    graph = hip::capture_end();
    if (!ok && graph) { hip::graph_destroy(graph); graph = nullptr; }
    return graph != nullptr;
  }
  // Go on at another position (after a prompt, or with another sequence).
  void seek(int64_t pos) {
    if (pos == cur_pos) return;
    cur_pos = pos;
    if (d_pos) {
      hip::flush();
      hip::upload_u32(d_pos, (unsigned)pos);
    }
  }
  // Feed token `id` at the current position without reading a token back.
  bool feed(M& m, int64_t id) {
    if (cur_pos >= max_ctx || !stage_embed(m, id)) return false;
    bool ok;
    if (graph) ok = hip::graph_launch(graph);
    else ok = step_layers(m, cur_pos);
    cur_pos++;
    return ok;
  }
  // One decode step: feed + greedy token (-1 when the cache is full or a launch failed).
  int64_t step(M& m, int64_t id) {
    if (!feed(m, id)) return -1;
    int64_t idx = -1;
    return hip::argmax(logits_device(m), vocab_size(m), &idx) ? idx : -1;
  }
  // Replays advance only the device counter; bring the host cache position up to date
  // before switching to a host-position call.
  void sync_host_pos(M& m) const {
    if (graph) set_cache_pos(m, cur_pos);
  }
  bool ok() const { return graph != nullptr; }
  void destroy() {
    if (graph) hip::graph_destroy(graph);
    if (d_pos) hip::release(d_pos, 0, nullptr);
    graph = nullptr;
    d_pos = nullptr;
  }
};

// One sequence at a time through a model: tokens in portions of any size (a single token by the
// recorded decode step, more as prompt chunks), logits where they are asked for, greedy generation.
template <class M>
class sequence {
  M& m_;
  captured_decoder<M> dec_;
  bool tried_ = false;              // recording was tried (it may not be offered)
  void *rows_ = nullptr, *idx_ = nullptr, *out_ = nullptr;   // rows whose logits are asked for
  float *idx_host_ = nullptr, *out_host_ = nullptr;
  int64_t cap_ = 0;

  bool room(int64_t n) {
    if (n <= cap_) return true;
    release();
    rows_ = hip::alloc_device(n * chunk_row_width(m_) * 4);
    idx_ = hip::alloc(n * 4, &idx_host_);
    out_ = hip::alloc(n * vocab_size(m_) * 4, &out_host_);
    cap_ = rows_ && idx_ && out_ ? n : 0;
    return cap_ > 0;
  }
  void release() {
    for (void** b : {&rows_, &idx_, &out_}) {
      if (*b) hip::release(*b, 0, nullptr);
      *b = nullptr;
    }
    cap_ = 0;
  }
  // logits of rows want[0..n) of the chunk just run
  bool rows_logits(const int64_t* want, int64_t n, int64_t T, float* out) {
    const int64_t V = vocab_size(m_), step = 256;
    for (int64_t w0 = 0; w0 < n; w0 += step) {
      const int64_t k = std::min(step, n - w0);
      if (!room(std::min(step, n))) return false;
      for (int64_t i = 0; i < k; i++) reinterpret_cast<int32_t*>(idx_host_)[i] = (int32_t)want[w0 + i];
      hip::upload(idx_, idx_host_, k);
      bool ok = hip::gather_rows(chunk_rows(m_), idx_, rows_, chunk_row_width(m_), k, T);
      ok = ok && (k == 1 ? gemv(head(m_), rows_, out_) : gemm(head(m_), rows_, out_, k));
      if (!ok) return false;
      hip::flush();
      if (!hip::download_raw(out + w0 * V, out_, k * V * 4)) return false;
    }
    return true;
  }

 public:
  explicit sequence(M& m) : m_(m) {}
  sequence(const sequence&) = delete;
  sequence& operator=(const sequence&) = delete;
  ~sequence() {
    dec_.destroy();
    release();
  }
  int64_t pos() const { return cache_pos(m_); }
  void reset() { set_cache_pos(m_, 0); }

  // The next n tokens; `want` lists (ascending) which of them get logits, [n_want, vocab] into out.
  bool feed(const int64_t* tokens, int64_t n, const int64_t* want, int64_t n_want, float* out, int64_t chunk = 512) {
    const int64_t p = pos(), V = vocab_size(m_);
    if (n <= 0 || n_want < 0 || chunk <= 0 || p + n > context_capacity(m_)) return false;
    for (int64_t i = 0; i < n_want; i++)
      if (want[i] < 0 || want[i] >= n || (i && want[i] <= want[i - 1])) return false;
    for (int64_t i = 0; i < n; i++)
      if (tokens[i] < 0 || tokens[i] >= V) return false;
    if (n == 1) {
      if (!tried_) {
        tried_ = true;
        dec_.init(m_, tokens[0], p);
      }
      dec_.seek(p);
      if (!dec_.feed(m_, tokens[0])) return false;
      set_cache_pos(m_, p + 1);
      if (n_want) std::copy(logits(m_), logits(m_) + V, out);
      return true;
    }
    if (longest_chunk(m_) > 0) chunk = std::min(chunk, longest_chunk(m_));
    int64_t w = 0;
    for (int64_t t0 = 0; t0 < n; t0 += chunk) {
      const int64_t T = std::min(chunk, n - t0);
      if (!prompt_chunk(m_, tokens + t0, T)) return false;
      std::vector<int64_t> here;
      const int64_t w0 = w;
      for (; w < n_want && want[w] < t0 + T; w++) here.push_back(want[w] - t0);
      if (!here.empty() && !rows_logits(here.data(), (int64_t)here.size(), T, out + w0 * V)) return false;
    }
    return true;
  }

  // Greedy continuation: n new tokens after the last fed token's successor `next` (the argmax of its
  // logits); the loop runs on the device. Returns how many were generated into out.
  int64_t generate(int64_t next, int64_t n, int32_t* out) {
    const int64_t p = pos();
    greedy_loop<M> g;
    int64_t done = 0;
    if (n > 0 && p < context_capacity(m_) && g.init(m_, next, p)) {
      done = g.run(n);
      const int32_t* t = g.tokens();
      std::copy(t + p, t + p + done, out);
      g.sync_host_pos(m_);
    }
    g.destroy();
    return done;
  }
};

}  // namespace loops
}  // namespace tl
