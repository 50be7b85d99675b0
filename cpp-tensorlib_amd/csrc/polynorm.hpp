// A cubic whose powers are each scaled to unit mean square over a row of ff values (tlhip_polynorm).
#pragma once

#include "common.hpp"

namespace tlhip {

struct PolySums {
  float s2 = 0.f, s4 = 0.f, s6 = 0.f;
  __device__ __forceinline__ void add(float v) {
    const float v2 = v * v, v4 = v2 * v2;
    s2 += v2;
    s4 += v4;
    s6 = fmaf(v4, v2, s6);
  }
  __device__ __forceinline__ void add(const float4 v) { add(v.x); add(v.y); add(v.z); add(v.w); }
};
struct PolyCoef {
  float r1, r2, r3, e;
  __device__ __forceinline__ float operator()(float v) const { return fmaf(fmaf(fmaf(r3, v, r2), v, r1), v, e); }
};
// The block's sums -> the row's coefficients, in every thread. red: 3 * NT / 64 floats of LDS.
template <int NT>
__device__ __forceinline__ PolyCoef poly_coef(const tlhip_polynorm& p, PolySums s, float* red) {
  constexpr int NW = NT / 64;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  s.s2 = wave_sum(s.s2);
  s.s4 = wave_sum(s.s4);
  s.s6 = wave_sum(s.s6);
  if (lane == 0) { red[wave] = s.s2; red[NW + wave] = s.s4; red[2 * NW + wave] = s.s6; }
  __syncthreads();
  s.s2 = s.s4 = s.s6 = 0.f;
#pragma unroll
  for (int w = 0; w < NW; w++) { s.s2 += red[w]; s.s4 += red[NW + w]; s.s6 += red[2 * NW + w]; }
  const float inv = 1.0f / (float)p.ff;
  return PolyCoef{p.c1 / sqrtf(s.s2 * inv + p.eps), p.c2 / sqrtf(s.s4 * inv + p.eps), p.c3 / sqrtf(s.s6 * inv + p.eps), p.c0};
}

// Elements [i0, i1) of one row by a block of NT threads; the three means are taken over the whole row
// by every block that works on it.
template <int NT>
__device__ __forceinline__ void polynorm_block(const tlhip_polynorm& p, const float* __restrict__ z, float* __restrict__ y,
                                               int i0, int i1, float* red) {
  const int tid = threadIdx.x, ff = (int)p.ff, n4 = ff >> 2;
  PolySums s;
  for (int i = tid; i < n4; i += NT) s.add(reinterpret_cast<const float4*>(z)[i]);
  for (int i = 4 * n4 + tid; i < ff; i += NT) s.add(z[i]);
  const PolyCoef f = poly_coef<NT>(p, s, red);
  for (int i = i0 + tid; i < i1; i += NT) y[i] = f(z[i]);
}

// A whole row whose values stay in registers: ff a multiple of 4 up to 4 * NT * L, z and y 16-byte aligned.
template <int NT, int L>
__device__ __forceinline__ void polynorm_row(const tlhip_polynorm& p, const float* __restrict__ z, float* __restrict__ y,
                                             float* red) {
  const int tid = threadIdx.x, n4 = (int)p.ff >> 2;
  float4 v[L];
  PolySums s;
#pragma unroll
  for (int k = 0; k < L; k++) {
    const int i = tid + k * NT;
    v[k] = reinterpret_cast<const float4*>(z)[min(i, n4 - 1)];
  }
#pragma unroll
  for (int k = 0; k < L; k++)
    if (tid + k * NT < n4) s.add(v[k]);
  const PolyCoef f = poly_coef<NT>(p, s, red);
#pragma unroll
  for (int k = 0; k < L; k++) {
    const int i = tid + k * NT;
    if (i < n4) reinterpret_cast<float4*>(y)[i] = make_float4(f(v[k].x), f(v[k].y), f(v[k].z), f(v[k].w));
  }
}

int check_polynorm(const tlhip_polynorm* p, const char* who);
}  // namespace tlhip
