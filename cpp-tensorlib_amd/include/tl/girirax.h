#pragma once

// The Girirax decoder on tl::hip: state-space layers (Mamba-2) and latent-attention layers in any order, a gated
// GELU feed-forward with biases behind either, and norms on what a sublayer writes instead of on what it reads,
//   x += m rms(mixer(x)) w1;   x += m rms(mlp(x)) w2.
//
// A sublayer reads the residual itself, so the norm of one sublayer's output, its bias and the residual sum are
// the staging pass of the next sublayer's first product (m folded into the weights w). Decode, per layer:
//   state space       [sum -> in] , [step] , [group norm -> o] , [sum -> gate|up, gelu] , [down]
//   latent attention  [sum -> dq|dkv|gate] , [norm -> uq] , [query, cache row] , [attend] , [join, uv, gate] , [o] , ...
//
// Residual, norms, scores, decays, step sizes and state are f32; weights stay the bf16 of the file; the latent
// cache holds one bf16 per number, or, in the exact form, three that add up to the f32.
//
// Columns and rows are padded with zero weights where the kernels want whole vectors (products' K and the
// width to 32); a norm over a padded row has its constants adjusted so that it is the norm over the real one.

#include <algorithm>
#include <cmath>
#include <cstdint>
#include <cstring>
#include <map>
#include <stdexcept>
#include <string>
#include <utility>
#include <vector>

#include "decode_loop.h"
#include "hip.h"
#include "json.h"
#include "linear.h"
#include "model_source.h"

namespace tl {
namespace girirax {

using namespace weights;

// ---- configuration ---------------------------------------------------------------------------
struct ssm_config {
  int64_t heads = 0, state = 0, groups = 0, vdim = 0, taps = 0, norm_groups = 0;
};
struct latent_config {
  int64_t heads = 0, dim = 0, rot_dim = 0, vdim = 0, kv_rank = 0, q_rank = 0;
  double rot_base = 0;
  float scale = 1;
};
struct layer_config {
  bool attention = false;            // which of the two mixers
  ssm_config ssm;
  latent_config latent;
  int64_t ff = 0;                    // 0: no feed-forward
};
struct config {
  int64_t vocab = 0, width = 0;
  float eps = 0, embed_scale = 1, residual_mult = 1;
  std::vector<layer_config> layers;
};

constexpr const char* kArchitecture = "Girirax";

inline config parse_config(const json::value& j) {
  const auto require = [](bool ok, const std::string& what) {
    if (!ok) throw std::runtime_error("config: " + what);
  };
  config c;
  require(j.at("architecture").str() == kArchitecture, "another architecture");
  c.vocab = j.at("vocab").integer();
  c.width = j.at("width").integer();
  c.eps = (float)j.at("norm").at("eps").num();
  c.embed_scale = (float)j.at("embedding").at("scale").num();
  c.residual_mult = (float)j.at("residual_mult").num();
  require(c.vocab > 0 && c.width > 0 && c.eps >= 0, "bad vocab, width or eps");
  for (const json::value& l : j.at("layers").items()) {
    const std::string where = "layer " + std::to_string(c.layers.size());
    const json::value& m = l.at("mixer");
    const std::string& type = l.at("type").str();
    layer_config n;
    if (type == "mamba2") {
      ssm_config& s = n.ssm;
      s.heads = m.at("heads").integer();
      s.state = m.at("state").integer();
      s.groups = m.at("groups").integer();
      s.vdim = m.at("vdim").integer();
      s.taps = m.at("conv").integer();
      s.norm_groups = m.at("norm_groups").integer();
      require(s.heads > 0 && s.state > 0 && s.groups > 0 && s.heads % s.groups == 0 && s.vdim > 0 && s.taps > 0 &&
                  s.norm_groups > 0 && s.heads * s.vdim % s.norm_groups == 0,
              where + ": bad state-space sizes");
    } else if (type == "latent_attention") {
      n.attention = true;
      latent_config& a = n.latent;
      a.heads = m.at("heads").integer();
      a.dim = m.at("dim").integer();
      a.rot_dim = m.at("rot_dim").integer();
      a.vdim = m.at("vdim").integer();
      a.kv_rank = m.at("kv_rank").integer();
      a.q_rank = m.at("q_rank").integer();
      a.scale = (float)m.at("scale").num();
      a.rot_base = m.at("rot").at("base").num();
      require(a.heads > 0 && a.dim > 0 && a.rot_dim >= 0 && a.rot_dim % 2 == 0 && a.vdim > 0 && a.kv_rank > 0 && a.q_rank > 0 &&
                  a.rot_base > 0,
              where + ": bad attention sizes");
      require(m.at("rot").at("dims").integer() == a.rot_dim, where + ": the whole rotated part turns, so rot.dims must be rot_dim");
    } else {
      require(false, where + ": unknown mixer");
    }
    const json::value* f = l.find("mlp");
    if (f && !f->is_null()) {
      require(f->at("kind").str() == "dense", where + ": unknown feed-forward");
      n.ff = f->at("ff").integer();
      require(n.ff > 0, where + ": bad feed-forward size");
    }
    c.layers.push_back(n);
  }
  require(!c.layers.empty(), "no layers");
  return c;
}

// ---- model -----------------------------------------------------------------------------------
struct layer {
  bool attention = false;
  linear win, uq, wout;              // uq: attention only
  hip::ssm ss;
  hip::latent_attn la;
  int64_t q_off = 0;                 // columns of u that hold the query latent
  void* q_norm = nullptr;            // over the padded latent, with q_eps
  float q_eps = 0;
  void* y_norm = nullptr;            // state space: of the gated output, y_n entries in y_parts runs
  int64_t y_n = 0, y_parts = 0;
  void *norm1 = nullptr, *norm2 = nullptr;   // residual factor and padding folded in
  linear gate_up, down;
  void *gate_up_b = nullptr, *down_b = nullptr;
  bool mlp = false;
};
struct scratch {                     // one token
  void *tok = nullptr, *u = nullptr, *q = nullptr, *y = nullptr, *act = nullptr, *delta = nullptr, *h = nullptr, *cq = nullptr,
       *gu = nullptr, *logitsb = nullptr;
  void* res[2] = {nullptr, nullptr};
  float* logits_host = nullptr;
};
struct chunk_scratch {               // up to T tokens
  int64_t T = 0;
  void *tok = nullptr, *h = nullptr, *res = nullptr, *u = nullptr, *q = nullptr, *cq = nullptr, *y = nullptr, *gu = nullptr,
       *act = nullptr, *parts = nullptr;
  int64_t parts_bytes = 0;
  float* tok_host = nullptr;
};

struct model {
  config c;
  int64_t wp = 0;                    // width rounded up to 32
  float eps = 0;                     // norms over wp columns
  int64_t max_ctx = 0, max_chunk = 0, pos = 0;
  std::vector<layer> layers;
  void* onorm = nullptr;
  linear lm_head;                    // the embedding table, rows padded to wp
  scratch s;
  chunk_scratch ps;
  void* step_tok = nullptr;          // where the next step's token id lies on the device
  int64_t u_cols = 0, q_cols = 0, cq_cols = 0, y_cols = 0, ff_cols = 0;   // widest rows
  // true: sums, norms and activations inside the products that need them; false: one launch per op
  bool fused = true;
  // true: every product exact (bf16 weights times three exact terms of an activation, the latent cache in
  // three terms); false: large products on the backend's prepared f16 form of the weights, the cache in bf16.
  // Chosen before build().
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
// longest prompt chunk.
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
  const auto upload_f = [&](const std::vector<float>& v) { return upload(v.data(), (int64_t)v.size() * 4); };
  const auto floats = [&](const std::string& name, int64_t n) {
    std::vector<uint16_t> b((size_t)n);
    src.read(name, n, 0, b.data(), 1);
    std::vector<float> v((size_t)n);
    for (size_t i = 0; i < v.size(); i++) v[i] = bf16_to_f32(b[i]);
    return v;
  };
  // `name` [n] times f, padded with zeros to `to`
  const auto padded = [&](const std::string& name, int64_t n, int64_t to, double f = 1.0) {
    std::vector<float> v = floats(name, n);
    for (float& x : v) x = (float)((double)x * f);
    v.resize((size_t)to, 0.0f);
    return upload_f(v);
  };
  // projections stacked by rows; K: their columns, padded to KP
  const auto stack = [&](const std::vector<source::part>& parts, int64_t N, int64_t K, int64_t KP) {
    host.assign((size_t)(N * KP), 0);
    for (const auto& p : parts) src.read(p.name, p.rows, K, host.data() + p.at * KP, KP);
    return linear{upload(host.data(), N * KP * 2), N, KP, wfmt::bf16_row};
  };
  // (cos, sin) of every position, one table per (dims, base)
  std::map<std::pair<int64_t, double>, void*> tables;
  const auto angles = [&](int64_t dims, double base, int64_t capacity) -> void* {
    void*& t = tables[{dims, base}];
    if (!t) {
      std::vector<float> v((size_t)(capacity * dims) + 2, 0.0f);
      for (int64_t i = 0; i < dims / 2; i++) {
        const double f = std::pow(base, -2.0 * (double)i / (double)dims);
        for (int64_t p = 0; p < capacity; p++) {
          v[(size_t)(p * dims + 2 * i)] = (float)std::cos((double)p * f);
          v[(size_t)(p * dims + 2 * i + 1)] = (float)std::sin((double)p * f);
        }
      }
      t = upload_f(v);
    }
    return t;
  };
  const double pad_gain = std::sqrt((double)E / (double)WP), m = cfg.residual_mult;

  M.layers.assign(cfg.layers.size(), layer{});
  M.u_cols = M.q_cols = M.cq_cols = M.y_cols = M.ff_cols = 0;
  for (size_t i = 0; i < cfg.layers.size(); i++) {
    const layer_config& lc = cfg.layers[i];
    layer& L = M.layers[i];
    const std::string p = "l" + std::to_string(i) + ".", pm = p + "mix.", pf = p + "mlp.";
    L.attention = lc.attention;
    int64_t ny;
    if (!lc.attention) {
      const ssm_config& sc = lc.ssm;
      hip::ssm& s = L.ss;
      s.heads = sc.heads; s.state = sc.state; s.groups = sc.groups; s.vdim = sc.vdim; s.taps = sc.taps;
      const int64_t inner = sc.heads * sc.vdim, ch = inner + 2 * sc.groups * sc.state;
      s.z_off = 0;                   // rows of the file's matrix: z | x | B | C | dt
      s.x_off = inner;
      s.dt_off = inner + ch;
      s.y_off = 0;
      const int64_t rows = inner + ch + sc.heads;
      L.win = stack({{pm + "in", rows, 0}}, up(rows, 8), E, WP);
      std::vector<uint16_t> w((size_t)(ch * sc.taps));
      src.read(pm + "conv", ch, sc.taps, w.data(), sc.taps);
      std::vector<float> wt(w.size());
      for (int64_t c = 0; c < ch; c++)
        for (int64_t k = 0; k < sc.taps; k++) wt[(size_t)(k * ch + c)] = bf16_to_f32(w[(size_t)(c * sc.taps + k)]);
      s.conv_w = upload_f(wt);
      s.conv_b = upload_f(floats(pm + "conv.b", ch));
      s.dt_bias = upload_f(floats(pm + "dt_bias", sc.heads));
      std::vector<float> dec = floats(pm + "A_log", sc.heads);
      for (float& x : dec) x = (float)(-std::exp((double)x) * 1.4426950408889634);
      s.decay = upload_f(dec);
      s.skip = upload_f(floats(pm + "D", sc.heads));
      s.conv_state = M.keep(hip::alloc_zeros(hip::ssm_conv_bytes(s)));
      s.ssm_state = M.keep(hip::alloc_zeros(hip::ssm_state_bytes(s)));
      ny = inner;
      L.y_n = inner;
      L.y_parts = sc.norm_groups;
      L.y_norm = padded(pm + "norm", inner, up(inner, 32));
    } else {
      const latent_config& ac = lc.latent;
      hip::latent_attn& a = L.la;
      a.heads = ac.heads; a.dim = ac.dim; a.rot_dim = ac.rot_dim; a.vdim = ac.vdim; a.kv_rank = ac.kv_rank;
      a.scale = ac.scale;
      a.eps = cfg.eps;
      a.capacity = up(max_ctx, 32);
      a.planes = M.exact ? 3 : 1;
      const int64_t qp = up(ac.q_rank, 32), kp = up(ac.kv_rank, 8);
      L.q_off = 0;
      a.kv_off = qp;
      a.gate_off = qp + up(ac.kv_rank + ac.rot_dim, 8);
      a.y_off = 0;
      const int64_t rows = a.gate_off + up(ac.heads * ac.vdim, 8);
      L.win = stack({{pm + "dq", ac.q_rank, 0}, {pm + "dkv", ac.kv_rank + ac.rot_dim, a.kv_off}, {pm + "g", ac.heads * ac.vdim, a.gate_off}},
                    rows, E, WP);
      L.q_norm = padded(pm + "dq.norm", ac.q_rank, qp, std::sqrt((double)ac.q_rank / (double)qp));
      L.q_eps = (float)((double)cfg.eps * (double)ac.q_rank / (double)qp);
      const int64_t nq = ac.heads * (ac.dim + ac.rot_dim);
      L.uq = stack({{pm + "uq", nq, 0}}, up(nq, 8), ac.q_rank, qp);
      a.kv_norm = upload_f(floats(pm + "dkv.norm", ac.kv_rank));
      a.uk = stack({{pm + "uk", ac.heads * ac.dim, 0}}, ac.heads * ac.dim, ac.kv_rank, kp).w;
      a.uv = stack({{pm + "uv", ac.heads * ac.vdim, 0}}, ac.heads * ac.vdim, ac.kv_rank, kp).w;
      a.angles = angles(ac.rot_dim, ac.rot_base, a.capacity);
      a.keys = M.keep(hip::alloc_zeros(hip::latent_cache_bytes(a, false)));
      a.values = M.keep(hip::alloc_zeros(hip::latent_cache_bytes(a, true)));
      ny = ac.heads * ac.vdim;
      M.q_cols = std::max(M.q_cols, L.uq.N);
      M.cq_cols = std::max(M.cq_cols, qp);
    }
    const int64_t kp = up(ny, 32);
    host.assign((size_t)(WP * kp), 0);
    src.read(pm + "o", E, ny, host.data(), kp);
    L.wout = linear{upload(host.data(), WP * kp * 2), WP, kp, wfmt::bf16_row};
    L.norm1 = padded(p + "norm1", E, WP, m * pad_gain);
    M.u_cols = std::max(M.u_cols, L.win.N);
    M.y_cols = std::max(M.y_cols, kp);

    L.mlp = lc.ff > 0;
    if (L.mlp) {
      const int64_t fp = up(lc.ff, 32);
      L.gate_up = stack({{pf + "gate", lc.ff, 0}, {pf + "up", lc.ff, fp}}, 2 * fp, E, WP);
      std::vector<float> b = floats(pf + "gate.b", lc.ff), b2 = floats(pf + "up.b", lc.ff);
      b.resize((size_t)fp, 0.0f);
      b2.resize((size_t)fp, 0.0f);
      b.insert(b.end(), b2.begin(), b2.end());
      L.gate_up_b = upload_f(b);
      host.assign((size_t)(WP * fp), 0);
      src.read(pf + "down", E, lc.ff, host.data(), fp);
      L.down = linear{upload(host.data(), WP * fp * 2), WP, fp, wfmt::bf16_row};
      L.down_b = padded(pf + "down.b", E, WP);
      L.norm2 = padded(p + "norm2", E, WP, m * pad_gain);
      M.ff_cols = std::max(M.ff_cols, fp);
    }
  }
  M.onorm = padded("final.norm", E, WP, pad_gain);
  M.lm_head = stack({{"embed", cfg.vocab, 0}}, cfg.vocab, E, WP);

  scratch& S = M.s;
  const auto A = [&](int64_t k) { return M.keep(hip::alloc_zeros(std::max<int64_t>(k, 4) * 4)); };
  S.tok = M.keep(hip::alloc(4, nullptr));
  S.res[0] = A(WP);
  S.res[1] = A(WP);
  S.h = A(WP);
  S.delta = A(WP);
  S.u = A(M.u_cols);
  S.q = A(M.q_cols);
  S.cq = A(M.cq_cols);
  S.y = A(M.y_cols);                 // (columns past a layer's own meet zero weights: finite is enough)
  S.act = A(M.ff_cols);
  S.gu = A(2 * M.ff_cols);
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
inline void load_random(model& M, const json::value& cfg, uint32_t seed, int64_t max_ctx, int64_t chunk = 512) {
  source::random src(seed, 0);
  build(M, parse_config(cfg), src, max_ctx, chunk);
}

// ---- one token -------------------------------------------------------------------------------
inline bool run_layers(model& M, int64_t pos, void* d_pos) {
  scratch& S = M.s;
  const int64_t WP = M.wp;
  bool ok = hip::embed_scaled(M.lm_head.w, WP, M.step_tok, S.res[0], 1, M.c.width, WP, M.c.vocab, M.c.embed_scale);
  int at = 0;                        // x is res[at], plus, where `norm` is set, the normed delta
  void *norm = nullptr, *bias = nullptr;
  // x brought up to date on the way into a product, or ahead of it
  const auto settle = [&]() {
    if (!norm) return true;
    const bool r = hip::postnorm_res_parts(S.res[at], S.delta, 1, bias, norm, S.res[at ^ 1], WP, M.eps);
    at ^= 1;
    norm = nullptr;
    return r;
  };
  const auto product = [&](const linear& w, void* y) {
    if (!norm || !M.fused) return settle() && gemv(w, S.res[at], y);
    const bool r = gemv_postnorm(w, S.res[at], S.delta, bias, norm, WP, 1, S.res[at ^ 1], y, M.eps);
    at ^= 1;
    norm = nullptr;
    return r;
  };
  for (layer& L : M.layers) {
    ok = ok && product(L.win, S.u);
    if (!L.attention) {
      ok = ok && hip::ssm_step(S.u, S.y, L.ss, pos, d_pos);
      if (M.fused)
        ok = ok && gemv_postnorm(L.wout, nullptr, S.y, nullptr, L.y_norm, L.y_n, L.y_parts, nullptr, S.delta, M.c.eps);
      else
        ok = ok && hip::rms_rows(S.y, L.wout.K, L.y_norm, S.y, L.wout.K, L.y_n, L.wout.K, L.y_parts, M.c.eps, 1) && gemv(L.wout, S.y, S.delta);
    } else {
      if (M.fused)
        ok = ok && gemv_rmsnorm(L.uq, S.u, nullptr, L.q_norm, nullptr, S.q, L.q_eps);
      else
        ok = ok && hip::rms_rows(S.u, L.win.N, L.q_norm, S.cq, L.uq.K, L.uq.K, L.uq.K, 1, L.q_eps, 1) && gemv(L.uq, S.cq, S.q);
      ok = ok && hip::latent_attn_run(S.u, L.win.N, S.q, L.uq.N, S.y, L.wout.K, L.la, 1, pos, d_pos) && gemv(L.wout, S.y, S.delta);
    }
    norm = L.norm1;
    bias = nullptr;
    if (L.mlp) {
      if (M.fused) {
        ok = ok && gemv_postnorm_geglu(L.gate_up, S.res[at], S.delta, bias, norm, S.res[at ^ 1], L.gate_up_b, S.act, M.eps);
        at ^= 1;
      } else {
        ok = ok && settle() && gemv(L.gate_up, S.res[at], S.gu) && hip::geglu_rows(S.gu, L.gate_up_b, S.act, L.down.K, 1);
      }
      ok = ok && gemv(L.down, S.act, S.delta);
      norm = L.norm2;
      bias = L.down_b;
    }
  }
  ok = ok && settle();
  if (M.fused) return ok && gemv_rmsnorm(M.lm_head, S.res[at], nullptr, M.onorm, nullptr, S.logitsb, M.eps);
  return ok && hip::rmsnorm(S.res[at], M.onorm, S.h, WP, M.eps) && gemv(M.lm_head, S.h, S.logitsb);
}

// ---- prompt chunks ---------------------------------------------------------------------------
inline bool reserve_chunk(model& M, int64_t T) {
  chunk_scratch& P = M.ps;
  if (T <= 0 || T > M.max_chunk) return false;
  if (P.T >= T) return true;
  const int64_t rows = M.max_chunk, WP = M.wp;   // once, for the longest
  const auto A = [&](int64_t k) { return M.keep(hip::alloc_zeros(std::max<int64_t>(k, 4) * 4)); };
  try {
    P.tok = M.keep(hip::alloc(rows * 4, &P.tok_host));
    P.h = A(rows * WP);
    P.res = A(rows * WP);
    P.u = A(rows * M.u_cols);
    P.q = A(rows * M.q_cols);
    P.cq = A(rows * M.cq_cols);
    P.y = A(rows * M.y_cols);
    P.gu = A(rows * 2 * M.ff_cols);
    P.act = A(rows * M.ff_cols);
    P.parts_bytes = 16 * rows * WP * 4;          // the GEMM splits K at most 16 ways
    P.parts = M.keep(hip::alloc_device(P.parts_bytes));
  } catch (const std::exception&) {
    return false;
  }
  P.T = rows;
  return true;
}

// layer_out (may be nullptr): [layers][T][width], the residual after every layer (diagnostics).
inline bool chunk_layers(model& M, int64_t T, float* layer_out = nullptr) {
  chunk_scratch& P = M.ps;
  const int64_t WP = M.wp, E = M.c.width, pos0 = M.pos;
  hip::set_prompt_f16(!M.exact);
  bool ok = hip::embed_scaled(M.lm_head.w, WP, P.tok, P.res, T, E, WP, M.c.vocab, M.c.embed_scale);
  std::vector<float> rows;
  for (size_t i = 0; i < M.layers.size() && ok; i++) {
    layer& L = M.layers[i];
    const int64_t ldu = L.win.N, ldy = L.wout.K, next = i + 1 < M.layers.size() ? M.layers[i + 1].win.N : 0;
    int np = 0;
    ok = gemm(L.win, P.res, P.u, T);
    if (!L.attention) {
      ok = ok && hip::ssm_chunk(P.u, ldu, P.y, ldy, L.ss, T, pos0) &&
           hip::rms_rows(P.y, ldy, L.y_norm, P.y, ldy, L.y_n, ldy, L.y_parts, M.c.eps, T);
    } else {
      ok = ok && hip::rms_rows(P.u, ldu, L.q_norm, P.cq, L.uq.K, L.uq.K, L.uq.K, 1, L.q_eps, T) && gemm(L.uq, P.cq, P.q, T) &&
           hip::latent_attn_run(P.u, ldu, P.q, L.uq.N, P.y, ldy, L.la, T, pos0);
    }
    ok = ok && gemm_parts(L.wout, P.y, P.parts, P.parts_bytes, T, &np) &&
         hip::postnorm_res_parts(P.res, P.parts, np, nullptr, L.norm1, P.res, WP, M.eps, T, L.mlp ? L.gate_up.N : next);
    if (L.mlp)
      ok = ok && gemm(L.gate_up, P.res, P.gu, T) && hip::geglu_rows(P.gu, L.gate_up_b, P.act, L.down.K, T) &&
           gemm_parts(L.down, P.act, P.parts, P.parts_bytes, T, &np) &&
           hip::postnorm_res_parts(P.res, P.parts, np, L.down_b, L.norm2, P.res, WP, M.eps, T, next);
    if (ok && layer_out) {
      rows.resize((size_t)(T * WP));
      hip::flush();
      ok = hip::download_raw(rows.data(), P.res, T * WP * 4);
      for (int64_t t = 0; t < T; t++) std::copy_n(rows.data() + t * WP, E, layer_out + ((int64_t)i * T + t) * E);
    }
  }
  return ok && hip::rmsnorm(P.res, M.onorm, P.h, WP, M.eps, T);
}

// ---- what the decode loops (decode_loop.h) ask of a model ----------------------------------------
inline int64_t vocab_size(const model& M) { return M.c.vocab; }
inline int64_t context_capacity(const model& M) { return M.max_ctx; }
inline int64_t cache_pos(const model& M) { return M.pos; }
// Only 0 (a new sequence) and the position the caches have reached mean anything: states hold the end
// of a sequence, not its whole past.
inline void set_cache_pos(model& M, int64_t p) { M.pos = p; }
inline int64_t longest_chunk(const model& M) { return M.max_chunk; }
inline void* logits_device(model& M) { return M.s.logitsb; }
inline const float* logits_host(const model& M) { return M.s.logits_host; }
inline const linear& head(const model& M) { return M.lm_head; }
inline void* chunk_rows(model& M) { return M.ps.h; }
inline int64_t chunk_row_width(const model& M) { return M.wp; }
inline int64_t layer_runs(const model& M) { return (int64_t)M.layers.size(); }
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
inline bool reserve_device_steps(model& M, bool) { return !M.layers.empty() && hip::graph_available(); }
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

}  // namespace girirax
}  // namespace tl
