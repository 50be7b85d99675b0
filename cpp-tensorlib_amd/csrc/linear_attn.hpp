// Gated linear attention: what the decode step (hybrid_step.hip) and the prompt-chunk kernels
// (linear_attn.hip) share, and the decode step's block.
//
//   state row c <- a_c row_c + k_c v,   o = sum_c q_c row_c,   ln a_c = -softplus(-z_c) / tau
//
// Everything is f32. Decays are kept as base-2 logarithms.
#pragma once

#include "attn_window.hpp"

namespace tlhip {

// log2 of the decay, -log2(1 + e^-z) / tau, from e = e^-|z| <= 1. log2(1 + e) keeps e's
// relative accuracy down to the smallest e: with w = fl(1 + e), log2(w) e / (w - 1) undoes w's rounding.
__device__ __forceinline__ float log2_decay(float z, float inv_tau) {
  const float e = exp2_native(-fabsf(z) * kLog2e), w = 1.f + e;
  const float l = w == 1.f ? e * kLog2e : log2_native(w) * (e * __builtin_amdgcn_rcpf(w - 1.f));
  return -(fmaxf(-z, 0.f) * kLog2e + l) * inv_tau;
}
// z of channel `ch` (head * dim + d): the low-rank product and its bias
__device__ __forceinline__ float decay_logit(const tlhip_linear_attn& a, const float* __restrict__ low, int ch) {
  const uint16_t* w = static_cast<const uint16_t*>(a.a2) + (size_t)ch * a.rank;
  float z = 0.f;
  for (int r = 0; r < (int)a.rank; r++) z = fmaf(__uint_as_float((uint32_t)w[r] << 16), low[r], z);
  return z + static_cast<const float*>(a.bias)[ch];
}
__host__ __device__ inline int64_t linear_state_ld(int64_t vdim) { return (vdim + 3) & ~(int64_t)3; }

// Decode step of head h, one block of 512 threads. The state is read from the slot of `pos` and
// written to the other one; a thread owns one float4 column of every ng-th row.
__device__ __forceinline__ void linear_step_block(const tlhip_linear_attn& a, const float* __restrict__ u,
                                                  float* __restrict__ y, int pos, int h, float* smem) {
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int dim = (int)a.dim, vdim = (int)a.vdim, ld = (int)linear_state_ld(vdim), nv4 = ld >> 2;
  const int ng = 512 / nv4, v4 = tid % nv4, dg = tid / nv4;
  const bool live = dg < ng;
  float* qs = smem;               // [dim]
  float* ks = qs + dim;
  float* al = ks + dim;
  float* vs = al + dim;           // [ld]
  float* red = vs + ld + ((4 - (3 * dim + ld) % 4) & 3);   // [ng][ld], 16-byte aligned
  float* sums = red + 2048;       // [8]
  const size_t slot = (size_t)a.heads * dim * ld;
  const float* src = static_cast<const float*>(a.state) + (size_t)(pos & 1) * slot + (size_t)h * dim * ld;
  float* dst = static_cast<float*>(a.state) + (size_t)((pos + 1) & 1) * slot + (size_t)h * dim * ld;
  constexpr int PRE = 8;          // rows of this thread requested up front
  float4 st[PRE];
#pragma unroll
  for (int i = 0; i < PRE; i++) {
    const int d = dg + i * ng;
    st[i] = live && pos > 0 && d < dim ? *reinterpret_cast<const float4*>(src + (size_t)d * ld + 4 * v4)
                                       : make_float4(0.f, 0.f, 0.f, 0.f);
  }
  for (int d = tid; d < dim; d += 512) {
    const int ch = h * dim + d;
    qs[d] = u[a.q_off + ch] * a.q_scale;
    ks[d] = u[a.k_off + ch];
    al[d] = exp2_native(log2_decay(decay_logit(a, u + a.low_off, ch), 1.0f / a.tau));
  }
  for (int v = tid; v < ld; v += 512) vs[v] = v < vdim ? u[a.v_off + (int64_t)h * vdim + v] : 0.f;
  __syncthreads();
  float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
  if (live) {
    const float v0 = vs[4 * v4], v1 = vs[4 * v4 + 1], v2 = vs[4 * v4 + 2], v3 = vs[4 * v4 + 3];
    const auto row = [&](int d, float4 s) {
      const float w = al[d], k = ks[d], q = qs[d];
      s.x = fmaf(w, s.x, k * v0); s.y = fmaf(w, s.y, k * v1); s.z = fmaf(w, s.z, k * v2); s.w = fmaf(w, s.w, k * v3);
      *reinterpret_cast<float4*>(dst + (size_t)d * ld + 4 * v4) = s;
      o.x = fmaf(q, s.x, o.x); o.y = fmaf(q, s.y, o.y); o.z = fmaf(q, s.z, o.z); o.w = fmaf(q, s.w, o.w);
    };
#pragma unroll
    for (int i = 0; i < PRE; i++)
      if (dg + i * ng < dim) row(dg + i * ng, st[i]);
    for (int d = dg + PRE * ng; d < dim; d += ng)
      row(d, pos > 0 ? *reinterpret_cast<const float4*>(src + (size_t)d * ld + 4 * v4) : make_float4(0.f, 0.f, 0.f, 0.f));
    *reinterpret_cast<float4*>(red + dg * ld + 4 * v4) = o;
  }
  __syncthreads();
  // o[v] summed over the row groups, its mean square over vdim, norm and gate
  float ss = 0.f;
  for (int v = tid; v < vdim; v += 512) {
    float t = 0.f;
    for (int g = 0; g < ng; g++) t += red[g * ld + v];
    vs[v] = t;
    ss = fmaf(t, t, ss);
  }
  ss = wave_sum(ss);
  if (lane == 0) sums[wave] = ss;
  __syncthreads();
  float tot = 0.f;
#pragma unroll
  for (int w = 0; w < 8; w++) tot += sums[w];
  const float inv = 1.0f / sqrtf(tot / (float)vdim + a.eps);
  for (int v = tid; v < vdim; v += 512) {
    const int64_t ch = (int64_t)h * vdim + v;
    const float g = u[a.gate_off + ch];
    y[a.y_off + ch] = vs[v] * inv * static_cast<const float*>(a.norm)[v] * (g * sigmoid_f(g)) * a.out_scale;
  }
}

__host__ __device__ inline size_t linear_step_lds(int64_t dim, int64_t vdim) {
  return (size_t)(3 * dim + linear_state_ld(vdim) + 4 + 2048 + 8) * sizeof(float);
}

int check_linear_attn(const tlhip_linear_attn* a, const char* who);
}  // namespace tlhip
