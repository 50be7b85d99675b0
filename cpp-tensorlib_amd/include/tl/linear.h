#pragma once

// Linear weights resident on the device and the products over them, in the two formats the models
// use, with the fused forms the backend offers. Shared by every model.

#include <cstdint>
#include <cstring>

#include "hip.h"
#include "types.h"

namespace tl {
namespace weights {

// A linear weight resident on the device. q4: the reference's one-buffer layout
// [packed [N][K/2] | scales [N][K/32]] (types.h:25-31). bf16_row: [N][K] bf16,
// the layout gemv_bf16_row and gemm_bf16_nt share (cuda.h:765-841).
enum class wfmt { q4, bf16_row };
struct linear {
  void* w = nullptr;
  int64_t N = 0, K = 0;
  wfmt fmt = wfmt::q4;
  int64_t bytes() const { return fmt == wfmt::q4 ? q4_bytes(N, K) : N * K * 2; }
};

// y[N] = a[K] . W
inline bool gemv(const linear& L, void* a, void* y) {
  if (L.fmt == wfmt::q4) {
    void* scales = static_cast<char*>(L.w) + L.N * L.K / 2;
    return hip::gemv_q4(a, L.w, scales, y, L.N, L.K, kQ4Group);
  }
  return hip::gemv_bf16_row(a, L.w, y, L.N, L.K);
}

// y = W . (attention output merged from n_parts split partials)
inline bool gemv_attn(const linear& L, void* parts, int n_parts, int64_t heads, int64_t head_dim, void* y) {
  if (L.fmt == wfmt::q4)
    return hip::gemv_q4_attn(parts, n_parts, heads, head_dim, L.w, static_cast<char*>(L.w) + L.N * L.K / 2, y, L.N,
                             L.K, kQ4Group);
  return hip::gemv_bf16_row_attn(parts, n_parts, heads, head_dim, L.w, y, L.N, L.K);
}

// Prompt-chunk products, T rows at a time: out[T, N] = a[T, K] . W^T for either weight format
// (bf16 rows or int4); `_parts` leaves the K-split parts for the launch that consumes them,
// `_swiglu` takes the fused [gate | up] weight and writes the gated activation [T, N / 2].
inline bool gemm(const linear& L, void* a, void* out, int64_t T) {
  if (L.fmt == wfmt::q4)
    return hip::gemm_q4_nt(a, L.w, static_cast<char*>(L.w) + L.N * L.K / 2, out, T, L.N, L.K, kQ4Group);
  return hip::gemm_bf16_nt(a, L.w, out, T, L.N, L.K);
}
inline bool gemm_parts(const linear& L, void* a, void* parts, int64_t parts_bytes, int64_t T, int* n_parts) {
  if (L.fmt == wfmt::q4)
    return hip::gemm_q4_nt_parts(a, L.w, static_cast<char*>(L.w) + L.N * L.K / 2, parts, parts_bytes, T, L.N,
                                 L.K, n_parts, kQ4Group);
  return hip::gemm_bf16_nt_parts(a, L.w, parts, parts_bytes, T, L.N, L.K, n_parts);
}
inline bool gemm_swiglu(const linear& L, void* a, void* act, int64_t T) {
  if (L.fmt == wfmt::q4)
    return hip::gemm_q4_nt_swiglu(a, L.w, static_cast<char*>(L.w) + L.N * L.K / 2, act, T, L.N / 2, L.K,
                                  kQ4Group);
  return hip::gemm_bf16_nt_swiglu(a, L.w, act, T, L.N / 2, L.K);
}

// y = W . swiglu(gu)
inline bool gemv_swiglu(const linear& L, void* gu, void* y) {
  if (L.fmt == wfmt::q4) {
    void* scales = static_cast<char*>(L.w) + L.N * L.K / 2;
    return hip::gemv_q4_swiglu(gu, L.w, scales, y, L.N, L.K, kQ4Group);
  }
  return hip::gemv_bf16_row_swiglu(gu, L.w, y, L.N, L.K);
}
// s = x (+ delta) -> xout ; y = W . rmsnorm(s, norm_w)
inline bool gemv_rmsnorm(const linear& L, void* x, void* delta, void* norm_w, void* xout, void* y,
                         float eps) {
  if (L.fmt == wfmt::q4) {
    void* scales = static_cast<char*>(L.w) + L.N * L.K / 2;
    return hip::gemv_q4_rmsnorm(x, delta, norm_w, xout, L.w, scales, y, L.N, L.K, kQ4Group, eps);
  }
  return hip::gemv_bf16_row_rmsnorm(x, delta, norm_w, xout, L.w, y, L.N, L.K, eps);
}

// L = [gate rows | up rows]; s = x (+ delta) -> xout ; act = swiglu(gate . n, up . n), n = rmsnorm(s, norm_w)
inline bool gemv_rmsnorm_gateup(const linear& L, void* x, void* delta, void* norm_w, void* xout, void* act,
                                float eps) {
  if (L.fmt == wfmt::q4) {
    void* scales = static_cast<char*>(L.w) + L.N * L.K / 2;
    return hip::gemv_q4_rmsnorm_gateup(x, delta, norm_w, xout, L.w, scales, act, L.N, L.K, kQ4Group, eps);
  }
  return hip::gemv_bf16_row_rmsnorm_gateup(x, delta, norm_w, xout, L.w, act, L.N, L.K, eps);
}

// s = x (nullptr: 0) + rms(delta + bias) norm_w over `parts` runs of n -> xout ; y = W . s (bf16 rows)
inline bool gemv_postnorm(const linear& L, void* x, void* delta, void* bias, void* norm_w, int64_t n, int64_t parts, void* xout,
                          void* y, float eps) {
  return L.fmt == wfmt::bf16_row && hip::gemv_bf16_row_postnorm(x, delta, bias, norm_w, n, parts, xout, L.w, y, L.N, L.K, eps);
}
// L = [gate rows | up rows] with biases: act = gelu_tanh(gate . s + b) (up . s + b)
inline bool gemv_postnorm_geglu(const linear& L, void* x, void* delta, void* bias, void* norm_w, void* xout, void* gu_bias,
                                void* act, float eps) {
  return L.fmt == wfmt::bf16_row &&
         hip::gemv_bf16_row_postnorm_geglu(x, delta, bias, norm_w, xout, L.w, gu_bias, act, L.N, L.K, eps);
}

namespace detail {

inline void* dev_from_host(const void* src, int64_t bytes) {
  float* host = nullptr;
  void* n = hip::alloc(bytes, &host);
  if (!n) return nullptr;
  std::memcpy(host, src, (size_t)bytes);
  hip::upload(n, host, (bytes + 3) / 4);  // device copy current from now on
  return n;
}

}  // namespace detail
}  // namespace weights
}  // namespace tl
