#pragma once

// The Lusadra decoder on tl::hip: layers whose sublayers all read one norm and are added together,
//   h = norm(x);  x += left_scale attention(h) + right_scale linear_attention(h) + polynorm_mlp(h),
// sinusoidal positions added to the token rows, and a range of layers run several times over with
// state of its own for every pass.
//
// What all sublayers of a layer read is one vector, so a layer has ONE input product: the rows of all
// its projections (queries, keys, values, gates, the low-rank decay input, mlp up) stacked, giving a
// row u; and what they write is added up, so it has ONE output product over the row y of everything
// they produce, its weight [left o | right o | down] side by side along K. Between the two stand the
// mixers (hip::window_attn, hip::linear_attn, hip::polynorm), which read columns of u and write columns
// of y, the mixer scales folded into y. A decode layer is three launches:
//   [norm -> input product] , [attention | linear attention | polynorm] , [output product]
// (four where the window is cut into splits), the residual add riding on the next layer's norm.
//
// Residual, norms, scores, decays, state and sums are f32; weights stay the bf16 of the file.
//
// Columns and rows are padded with zero weights where the kernels want whole vectors (segments to 8,
// the output product's K and the width to 32); a norm over a padded width has its constants adjusted
// so that it is the norm over the real one.

#include <algorithm>
#include <cmath>
#include <cstdint>
#include <cstring>
#include <stdexcept>
#include <string>
#include <vector>

#include "decode_loop.h"
#include "hip.h"
#include "json.h"
#include "linear.h"
#include "model_source.h"

namespace tl {
namespace lusadra {

using namespace weights;

// ---- configuration ---------------------------------------------------------------------------
struct attn_config {
  int64_t heads = 0, kv_heads = 0, dim = 0, window = 0;
  float scale = 1, temp_coef = 0, temp_every = 0;
};
struct linear_config {
  int64_t heads = 0, dim = 0, vdim = 0;
  float tau = 1;
};
struct layer_config {
  attn_config left;
  linear_config right;
  float left_scale = 1, right_scale = 1;
  int64_t ff = 0;                    // 0: no feed-forward
};
struct config {
  int64_t vocab = 0, width = 0;
  float eps = 0;
  std::vector<layer_config> layers;
  int64_t loop_start = 0, loop_stop = 0, loop_times = 0;   // times 0: no loop
};

constexpr float kSlopeExp = 8.0f;    // the heads' distance slopes: powers 1, 2, .. of 2^(-kSlopeExp/heads)
constexpr const char* kArchitecture = "Lusadra";

inline config parse_config(const json::value& j) {
  const auto require = [](bool ok, const std::string& what) {
    if (!ok) throw std::runtime_error("config: " + what);
  };
  config c;
  require(j.at("architecture").str() == kArchitecture, "another architecture");
  c.vocab = j.at("vocab").integer();
  c.width = j.at("width").integer();
  c.eps = (float)j.at("norm").at("eps").num();
  require(c.vocab > 0 && c.width > 0 && c.eps >= 0, "bad vocab, width or eps");
  for (const json::value& l : j.at("layers").items()) {
    const std::string where = "layer " + std::to_string(c.layers.size());
    require(l.at("type").str() == "parallel", where + ": unknown mixer");
    const json::value &m = l.at("mixer"), &a = m.at("left"), &r = m.at("right");
    layer_config n;
    n.left.heads = a.at("heads").integer();
    n.left.kv_heads = a.at("kv_heads").integer();
    n.left.dim = a.at("dim").integer();
    n.left.window = a.at("mask").at("size").integer();
    n.left.scale = (float)a.at("scale").num();
    n.left.temp_coef = (float)a.at("q_temp").at("coef").num();
    n.left.temp_every = (float)a.at("q_temp").at("every").num();
    require(n.left.heads > 0 && n.left.kv_heads > 0 && n.left.heads % n.left.kv_heads == 0 && n.left.dim > 0 &&
                n.left.window > 0 && n.left.temp_every > 0,
            where + ": bad attention sizes");
    require(!a.find("vdim") || a.at("vdim").integer() == n.left.dim, where + ": the values are the keys, so vdim must be dim");
    n.right.heads = r.at("heads").integer();
    n.right.dim = r.at("dim").integer();
    n.right.vdim = r.at("vdim").integer();
    n.right.tau = (float)r.at("tau").num();
    require(n.right.heads > 0 && n.right.dim > 0 && n.right.vdim > 0 && n.right.tau > 0, where + ": bad linear attention sizes");
    n.left_scale = (float)m.at("left_scale").num();
    n.right_scale = (float)m.at("right_scale").num();
    const json::value* f = l.find("mlp");
    if (f && !f->is_null()) {
      require(f->at("kind").str() == "dense", where + ": unknown feed-forward");
      n.ff = f->at("ff").integer();
      require(n.ff > 0, where + ": bad feed-forward size");
    }
    c.layers.push_back(n);
  }
  require(!c.layers.empty(), "no layers");
  const json::value* lp = j.find("loop");
  if (lp && !lp->is_null()) {
    c.loop_start = lp->at("start").integer();
    c.loop_stop = lp->at("stop").integer();
    c.loop_times = lp->at("times").integer();
    require(c.loop_start >= 0 && c.loop_start < c.loop_stop && c.loop_stop <= (int64_t)c.layers.size() && c.loop_times > 0,
            "bad loop");
  }
  return c;
}

// ---- model -----------------------------------------------------------------------------------
struct layer {
  linear win, wout;                  // [u columns, padded width], [padded width, y columns]
  void* norm = nullptr;              // the norm's one number, once per padded column
  hip::window_attn at;               // offsets, sizes and constants; ring and state belong to a run
  hip::linear_attn la;
  hip::polynorm pn;
  bool mlp = false;
};
// One pass of a layer: its cache and state. enter >= 0: the first layer of pass number `enter` of the loop.
struct run {
  int64_t layer = 0, enter = -1;
  void *ring = nullptr, *state = nullptr;
};
struct scratch {                     // one token
  void *tok = nullptr, *emb = nullptr, *u = nullptr, *y = nullptr, *delta = nullptr, *logitsb = nullptr, *h = nullptr;
  void* res[2] = {nullptr, nullptr};
  void* partials = nullptr;          // of an attention whose window is cut into splits
  int64_t partials_bytes = 0;
  float* logits_host = nullptr;
};
struct chunk_scratch {               // up to T tokens
  int64_t T = 0;
  void *tok = nullptr, *emb = nullptr, *h = nullptr, *res = nullptr, *u = nullptr, *y = nullptr, *parts = nullptr;
  int64_t parts_bytes = 0;
  float* tok_host = nullptr;
};

struct model {
  config c;
  int64_t wp = 0;                    // width rounded up to 32
  float eps = 0;                     // norms over wp columns
  int64_t max_ctx = 0, max_chunk = 0, pos = 0;
  std::vector<layer> layers;
  std::vector<run> runs;
  void *embed = nullptr, *steps = nullptr, *onorm = nullptr;
  linear lm_head;
  scratch s;
  chunk_scratch ps;
  void* step_tok = nullptr;          // where the next step's token id lies on the device
  int64_t u_cols = 0, y_cols = 0;    // widest rows
  // true: the decode step's three launches per layer; false: one launch per op
  bool fused = true;
  // prompt chunks: every product exact (bf16 weights times three exact terms of an activation, attention
  // on the fp32 matrix pipe); false: large products on the backend's prepared f16 form of the weights and
  // attention on the 16-bit matrix cores, two rounded terms per f32 operand
  bool exact = false;
  std::vector<void*> owned;          // every device buffer, for destroy()

  model() = default;
  model(const model&) = delete;
  model& operator=(const model&) = delete;
  ~model() { destroy(); }
  void destroy() {
    for (void* p : owned) hip::release(p, 0, nullptr);
    owned.clear();
  }
  void* keep(void* p) {
    if (!p) throw std::runtime_error("out of device memory");
    owned.push_back(p);
    return p;
  }
};

// Allocates everything and fills the weights from `src`. max_ctx: the longest sequence; chunk: the
// longest prompt chunk (the key rings hold a window and a chunk).
inline void build(model& M, const config& cfg, source::reader& src, int64_t max_ctx, int64_t chunk = 512) {
  using source::up;
  if (!hip::available()) throw std::runtime_error(std::string("GPU backend unavailable: ") + hip::unavailable_reason());
  if (max_ctx <= 0 || chunk <= 0 || chunk > 65535) throw std::runtime_error("bad context or chunk length");
  M.c = cfg;
  M.wp = up(cfg.width, 32);
  M.eps = (float)((double)cfg.eps * (double)cfg.width / (double)M.wp);
  M.max_ctx = max_ctx;
  M.max_chunk = std::min(chunk, max_ctx);
  M.pos = 0;
  const int64_t E = cfg.width, WP = M.wp;
  std::vector<uint16_t> host;
  const auto upload = [&](const void* p, int64_t bytes) {
    void* d = M.keep(hip::alloc_device(up(bytes, 16)));
    if (!hip::upload_raw(d, p, bytes)) throw std::runtime_error("upload failed");
    return d;
  };
  const auto floats = [&](const std::string& name, int64_t n) {   // n 0: one number
    std::vector<uint16_t> b((size_t)std::max<int64_t>(n, 1));
    src.read(name, n, 0, b.data(), 1);
    std::vector<float> v(b.size());
    for (size_t i = 0; i < b.size(); i++) v[i] = bf16_to_f32(b[i]);
    return v;
  };
  const auto norm = [&](const std::string& name) {
    const float g = floats(name, 0)[0];
    std::vector<float> v((size_t)WP, 0.0f);
    std::fill(v.begin(), v.begin() + E, (float)((double)g * std::sqrt((double)E / (double)WP)));
    return upload(v.data(), WP * 4);
  };
  // projections stacked by rows
  const auto stack = [&](const std::vector<source::part>& parts, int64_t N) {
    host.assign((size_t)(N * WP), 0);
    for (const auto& p : parts) src.read(p.name, p.rows, E, host.data() + p.at * WP, WP);
    return linear{upload(host.data(), N * WP * 2), N, WP, wfmt::bf16_row};
  };
  // output projections side by side: part.rows = its columns, part.at = its first column
  const auto beside = [&](const std::vector<source::part>& parts, int64_t K) {
    host.assign((size_t)(WP * K), 0);
    for (const auto& p : parts) src.read(p.name, E, p.rows, host.data() + p.at, K);
    return linear{upload(host.data(), WP * K * 2), WP, K, wfmt::bf16_row};
  };

  M.layers.assign(cfg.layers.size(), layer{});
  M.u_cols = M.y_cols = 0;
  int64_t partials = 0;
  for (size_t i = 0; i < cfg.layers.size(); i++) {
    const layer_config& lc = cfg.layers[i];
    layer& L = M.layers[i];
    const std::string p = "l" + std::to_string(i) + ".", pl = p + "mix.left.", pr = p + "mix.right.";
    std::vector<source::part> in, out;
    int64_t nu = 0, ny = 0;
    const auto seg = [&](std::vector<source::part>& list, int64_t& end, const std::string& name, int64_t n) {
      const int64_t at = end;
      list.push_back({name, n, at});
      end = up(at + n, 8);
      return at;
    };
    hip::window_attn& a = L.at;
    a.heads = lc.left.heads; a.kv_heads = lc.left.kv_heads; a.dim = lc.left.dim; a.window = lc.left.window;
    a.scale = lc.left.scale; a.temp_coef = lc.left.temp_coef; a.temp_every = lc.left.temp_every;
    a.slope_exp = kSlopeExp;
    a.out_scale = lc.left_scale;
    a.ring_ld = hip::window_ring_ld(a.dim);
    if (a.ring_ld == 0) throw std::runtime_error(p + ": attention head size beyond what the kernels hold");
    a.ring_rows = std::min(up(a.window - 1 + M.max_chunk, 32), up(max_ctx, 32));
    a.q_off = seg(in, nu, pl + "q", a.heads * a.dim);
    a.k_off = seg(in, nu, pl + "k", a.kv_heads * a.dim);
    a.gate_off = seg(in, nu, pl + "g", a.heads * a.dim);
    a.y_off = seg(out, ny, pl + "o", a.heads * a.dim);
    partials = std::max(partials, hip::mix_partials_bytes(&a));

    hip::linear_attn& r = L.la;
    r.heads = lc.right.heads; r.dim = lc.right.dim; r.vdim = lc.right.vdim;
    r.rank = src.rows_of(pr + "a1");
    r.tau = lc.right.tau;
    r.eps = cfg.eps;
    r.q_scale = (float)(1.0 / std::sqrt((double)r.dim));
    r.out_scale = lc.right_scale;
    r.q_off = seg(in, nu, pr + "q", r.heads * r.dim);
    r.k_off = seg(in, nu, pr + "k", r.heads * r.dim);
    r.v_off = seg(in, nu, pr + "v", r.heads * r.vdim);
    r.gate_off = seg(in, nu, pr + "g", r.heads * r.vdim);
    r.low_off = seg(in, nu, pr + "a1", r.rank);
    r.y_off = seg(out, ny, pr + "o", r.heads * r.vdim);
    host.assign((size_t)(r.heads * r.dim * r.rank), 0);
    src.read(pr + "a2", r.heads * r.dim, r.rank, host.data(), r.rank);
    r.a2 = upload(host.data(), (int64_t)host.size() * 2);
    r.bias = upload(floats(pr + "a2.b", r.heads * r.dim).data(), r.heads * r.dim * 4);
    r.norm = upload(floats(pr + "norm", r.vdim).data(), r.vdim * 4);

    L.mlp = lc.ff > 0;
    if (L.mlp) {
      const std::vector<float> act = floats(p + "mlp.act", 4);
      hip::polynorm& n = L.pn;
      n.ff = lc.ff;
      n.c1 = act[0]; n.c2 = act[1]; n.c3 = act[2]; n.c0 = act[3];
      n.eps = cfg.eps;
      n.z_off = seg(in, nu, p + "mlp.up", lc.ff);
      n.y_off = seg(out, ny, p + "mlp.down", lc.ff);
    }
    ny = up(ny, 32);
    L.norm = norm(p + "norm1");
    L.win = stack(in, nu);
    L.wout = beside(out, ny);
    M.u_cols = std::max(M.u_cols, nu);
    M.y_cols = std::max(M.y_cols, ny);
  }

  // the order in which layers run, each pass with a cache and a state of its own
  M.runs.clear();
  const int64_t n = (int64_t)cfg.layers.size();
  const bool loop = cfg.loop_times > 0;
  const auto add = [&](int64_t i, int64_t enter) {
    const layer& L = M.layers[(size_t)i];
    run q;
    q.layer = i;
    q.enter = enter;
    q.ring = M.keep(hip::alloc_zeros(L.at.kv_heads * L.at.ring_rows * L.at.ring_ld * 4));
    q.state = M.keep(hip::alloc_zeros(hip::linear_state_bytes(L.la.heads, L.la.dim, L.la.vdim)));
    M.runs.push_back(q);
  };
  for (int64_t i = 0; i < (loop ? cfg.loop_start : n); i++) add(i, -1);
  for (int64_t t = 0; t < (loop ? cfg.loop_times : 0); t++)
    for (int64_t i = cfg.loop_start; i < cfg.loop_stop; i++) add(i, i == cfg.loop_start ? t : -1);
  for (int64_t i = loop ? cfg.loop_stop : n; i < n; i++) add(i, -1);

  if (loop) {
    std::vector<uint16_t> b((size_t)(cfg.loop_times * E));
    src.read("loop.step", cfg.loop_times, E, b.data(), E);
    std::vector<float> v((size_t)(cfg.loop_times * WP), 0.0f);
    for (int64_t t = 0; t < cfg.loop_times; t++)
      for (int64_t k = 0; k < E; k++) v[(size_t)(t * WP + k)] = bf16_to_f32(b[(size_t)(t * E + k)]);
    M.steps = upload(v.data(), (int64_t)v.size() * 4);
  }
  host.assign((size_t)(cfg.vocab * E), 0);
  src.read("embed", cfg.vocab, E, host.data(), E);
  M.embed = upload(host.data(), cfg.vocab * E * 2);
  M.onorm = norm("final.norm");
  M.lm_head = stack({{"head", cfg.vocab, 0}}, cfg.vocab);

  scratch& S = M.s;
  const auto A = [&](int64_t k) { return M.keep(hip::alloc_zeros(k * 4)); };
  S.tok = M.keep(hip::alloc(4, nullptr));
  S.emb = A(WP);
  S.res[0] = A(WP);
  S.res[1] = A(WP);
  S.h = A(WP);
  S.delta = A(WP);
  S.u = A(M.u_cols);
  S.y = A(M.y_cols);                 // (columns between segments meet zero weights: finite is enough)
  S.partials_bytes = partials;
  if (partials) S.partials = A(partials / 4);
  S.logitsb = M.keep(hip::alloc(cfg.vocab * 4, &S.logits_host));
  M.step_tok = S.tok;
  hip::flush();
}

// A folder with config.json and model.safetensors.
inline void load(model& M, const json::value& cfg, const std::string& dir, int64_t max_ctx, int64_t chunk = 512) {
  const safetensors::file f(dir + "/model.safetensors");
  source::file src(f);
  build(M, parse_config(cfg), src, max_ctx, chunk);
}
inline void load_random(model& M, const json::value& cfg, uint32_t seed, int64_t rank, int64_t max_ctx, int64_t chunk = 512) {
  source::random src(seed, rank);
  build(M, parse_config(cfg), src, max_ctx, chunk);
}

// ---- one token -------------------------------------------------------------------------------
inline bool run_layers(model& M, int64_t pos, void* d_pos) {
  scratch& S = M.s;
  const int64_t WP = M.wp;
  const auto vec = [&](int64_t t) { return static_cast<char*>(M.steps) + t * WP * 4; };
  bool ok = hip::embed_sinusoid(M.embed, M.step_tok, S.emb, 1, M.c.width, WP, M.c.vocab, pos, d_pos);
  void* x = S.emb;                   // residual entering the layer
  void* d = nullptr;                 // output of the previous layer, not yet added
  int at = 0;                        // which of res[] the next residual goes to
  for (const run& q : M.runs) {
    layer& L = M.layers[(size_t)q.layer];
    hip::window_attn a = L.at;
    hip::linear_attn r = L.la;
    a.ring = q.ring;
    r.state = q.state;
    const hip::polynorm* pn = L.mlp ? &L.pn : nullptr;
    if (q.enter >= 0) {              // x (+ what is not yet added) (+ the token row) + the pass's vector
      ok = ok && hip::residual_sum(x, d, 1, q.enter > 0 ? S.emb : nullptr, vec(q.enter), S.res[at], WP, 1);
      x = S.res[at];
      at ^= 1;
      d = nullptr;
    }
    if (M.fused) {
      ok = ok && gemv_rmsnorm(L.win, x, d, L.norm, d ? S.res[at] : nullptr, S.u, M.eps) &&
           hip::mix_step(S.u, S.y, &a, &r, pn, pos, d_pos, S.partials, S.partials_bytes);
    } else {
      ok = ok && (d ? hip::rmsnorm_res(x, d, L.norm, S.res[at], S.h, WP, M.eps) : hip::rmsnorm(x, L.norm, S.h, WP, M.eps)) &&
           gemv(L.win, S.h, S.u) &&
           hip::mix_step(S.u, S.y, &a, nullptr, nullptr, pos, d_pos, S.partials, S.partials_bytes) &&
           hip::mix_step(S.u, S.y, nullptr, &r, nullptr, pos, d_pos, nullptr, 0) &&
           (!pn || hip::mix_step(S.u, S.y, nullptr, nullptr, pn, pos, d_pos, nullptr, 0));
    }
    if (d) {
      x = S.res[at];
      at ^= 1;
    }
    ok = ok && gemv(L.wout, S.y, S.delta);
    d = S.delta;
  }
  if (M.fused) return ok && gemv_rmsnorm(M.lm_head, x, d, M.onorm, nullptr, S.logitsb, M.eps);
  return ok && hip::rmsnorm_res(x, d, M.onorm, S.res[at], S.h, WP, M.eps) && gemv(M.lm_head, S.h, S.logitsb);
}

// ---- prompt chunks ---------------------------------------------------------------------------
inline bool reserve_chunk(model& M, int64_t T) {
  chunk_scratch& P = M.ps;
  if (T <= 0 || T > M.max_chunk) return false;
  if (P.T >= T) return true;
  const int64_t rows = M.max_chunk, WP = M.wp;   // once, for the longest
  const auto A = [&](int64_t k) { return M.keep(hip::alloc_zeros(k * 4)); };
  try {
    P.tok = M.keep(hip::alloc(rows * 4, &P.tok_host));
    P.emb = A(rows * WP);
    P.h = A(rows * WP);
    P.res = A(rows * WP);
    P.u = A(rows * M.u_cols);
    P.y = A(rows * M.y_cols);
    P.parts_bytes = 16 * rows * WP * 4;          // the GEMM splits K at most 16 ways
    P.parts = M.keep(hip::alloc_device(P.parts_bytes));
  } catch (const std::exception&) {
    return false;
  }
  P.T = rows;
  return true;
}

// layer_out (may be nullptr): [runs][T][width], the residual after every layer run (diagnostics).
inline bool chunk_layers(model& M, int64_t T, float* layer_out = nullptr) {
  chunk_scratch& P = M.ps;
  const int64_t WP = M.wp, E = M.c.width, pos0 = M.pos;
  const auto vec = [&](int64_t t) { return static_cast<char*>(M.steps) + t * WP * 4; };
  hip::set_prompt_f16(!M.exact);
  bool ok = hip::embed_sinusoid(M.embed, P.tok, P.emb, T, E, WP, M.c.vocab, pos0);
  void* x = P.emb;
  int np = 0;                        // K-split parts of the previous layer's output, not yet added
  std::vector<float> rows;
  int64_t done = 0;
  for (const run& q : M.runs) {
    layer& L = M.layers[(size_t)q.layer];
    hip::window_attn a = L.at;
    hip::linear_attn r = L.la;
    a.ring = q.ring;
    r.state = q.state;
    const int64_t ldu = L.win.N, ldy = L.wout.K;
    if (q.enter >= 0) {
      ok = ok && hip::residual_sum(x, np ? P.parts : nullptr, np, q.enter > 0 ? P.emb : nullptr, vec(q.enter), P.res, WP, T) &&
           hip::rmsnorm(P.res, L.norm, P.h, WP, M.eps, T);
      x = P.res;
    } else if (np) {
      ok = ok && hip::rmsnorm_res_parts(x, P.parts, np, L.norm, P.res, P.h, WP, M.eps, T, L.win.N);
      x = P.res;
    } else {
      ok = ok && hip::rmsnorm(x, L.norm, P.h, WP, M.eps, T);
    }
    ok = ok && gemm(L.win, P.h, P.u, T) && hip::window_attn_chunk(P.u, ldu, P.y, ldy, a, T, pos0, M.exact) &&
         hip::linear_attn_chunk(P.u, ldu, P.y, ldy, r, T, pos0) &&
         (!L.mlp || hip::polynorm_rows(P.u, ldu, P.y, ldy, L.pn, T)) &&
         gemm_parts(L.wout, P.y, P.parts, P.parts_bytes, T, &np);
    if (ok && layer_out) {           // the sum that the next norm forms, written out
      rows.resize((size_t)(T * WP));
      ok = hip::residual_sum(x, P.parts, np, nullptr, nullptr, P.res, WP, T);
      x = P.res;
      np = 0;
      hip::flush();
      ok = ok && hip::download_raw(rows.data(), P.res, T * WP * 4);
      for (int64_t t = 0; t < T; t++) std::copy_n(rows.data() + t * WP, E, layer_out + (done * T + t) * E);
      done++;
    }
    if (!ok) return false;
  }
  return np ? hip::rmsnorm_res_parts(x, P.parts, np, M.onorm, P.res, P.h, WP, M.eps, T)
            : hip::rmsnorm(x, M.onorm, P.h, WP, M.eps, T);
}

// ---- what the decode loops (decode_loop.h) ask of a model ----------------------------------------
inline int64_t vocab_size(const model& M) { return M.c.vocab; }
inline int64_t context_capacity(const model& M) { return M.max_ctx; }
inline int64_t cache_pos(const model& M) { return M.pos; }
// Only 0 (a new sequence) and the position the caches have reached mean anything: rings and states
// hold the end of a sequence, not its whole past.
inline void set_cache_pos(model& M, int64_t p) { M.pos = p; }
inline int64_t longest_chunk(const model& M) { return M.max_chunk; }
inline void* logits_device(model& M) { return M.s.logitsb; }
inline const float* logits_host(const model& M) { return M.s.logits_host; }
inline const linear& head(const model& M) { return M.lm_head; }
inline void* chunk_rows(model& M) { return M.ps.h; }
inline int64_t chunk_row_width(const model& M) { return M.wp; }
inline int64_t layer_runs(const model& M) { return (int64_t)M.runs.size(); }
inline bool stage_embed(model& M, int64_t token) {
  if (token < 0 || token >= M.c.vocab) return false;
  hip::upload_u32(M.s.tok, (unsigned)token);
  M.step_tok = M.s.tok;
  return true;
}
inline bool step_layers(model& M, int64_t pos, void* d_pos = nullptr, bool advance = true) {
  return run_layers(M, pos, d_pos) && (!d_pos || !advance || hip::incr_u32(d_pos));
}
inline bool step_layers_from(model& M, void* d_tok, void* d_pos) {
  M.step_tok = d_tok;
  const bool ok = run_layers(M, 0, d_pos);
  M.step_tok = M.s.tok;
  return ok;
}
inline bool reserve_device_steps(model& M, bool) { return !M.runs.empty() && hip::graph_available(); }
inline bool stage_chunk(model& M, const int64_t* tokens, int64_t T) {
  if (!reserve_chunk(M, T)) return false;
  for (int64_t t = 0; t < T; t++) {
    if (tokens[t] < 0 || tokens[t] >= M.c.vocab) return false;
    reinterpret_cast<int32_t*>(M.ps.tok_host)[t] = (int32_t)tokens[t];
  }
  hip::upload(M.ps.tok, M.ps.tok_host, T);
  return true;
}
inline bool prompt_chunk(model& M, const int64_t* tokens, int64_t T) {
  if (M.pos + T > M.max_ctx || !stage_chunk(M, tokens, T) || !chunk_layers(M, T)) return false;
  M.pos += T;
  return true;
}

using loops::logits;
using loops::prefill;
using loops::step_greedy;

}  // namespace lusadra
}  // namespace tl
