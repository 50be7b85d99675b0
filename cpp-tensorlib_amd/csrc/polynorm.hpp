// y = a N(z) + b N(z^2) + c N(z^3) + e, N(w) = w / sqrt(mean(w^2) + eps) over a row of ff values.
#pragma once

#include "common.hpp"

namespace tlhip {

// Elements [i0, i1) of one row by a block of NT threads; the three means are taken over the whole row
// by every block that works on it. red: 3 * NT / 64 floats of LDS.
template <int NT>
__device__ __forceinline__ void polynorm_block(const tlhip_polynorm& p, const float* __restrict__ z, float* __restrict__ y,
                                               int i0, int i1, float* red) {
  constexpr int NW = NT / 64;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, ff = (int)p.ff;
  float s2 = 0.f, s4 = 0.f, s6 = 0.f;
  const auto add = [&](float v) {
    const float v2 = v * v, v4 = v2 * v2;
    s2 += v2;
    s4 += v4;
    s6 = fmaf(v4, v2, s6);
  };
  const int n4 = ff >> 2;
  for (int i = tid; i < n4; i += NT) {
    const float4 v = reinterpret_cast<const float4*>(z)[i];
    add(v.x); add(v.y); add(v.z); add(v.w);
  }
  for (int i = 4 * n4 + tid; i < ff; i += NT) add(z[i]);
  s2 = wave_sum(s2);
  s4 = wave_sum(s4);
  s6 = wave_sum(s6);
  if (lane == 0) { red[wave] = s2; red[NW + wave] = s4; red[2 * NW + wave] = s6; }
  __syncthreads();
  s2 = s4 = s6 = 0.f;
#pragma unroll
  for (int w = 0; w < NW; w++) { s2 += red[w]; s4 += red[NW + w]; s6 += red[2 * NW + w]; }
  const float inv = 1.0f / (float)ff;
  const float r1 = p.a / sqrtf(s2 * inv + p.eps), r2 = p.b / sqrtf(s4 * inv + p.eps), r3 = p.c / sqrtf(s6 * inv + p.eps);
  for (int i = i0 + tid; i < i1; i += NT) {
    const float v = z[i];
    y[i] = fmaf(fmaf(fmaf(r3, v, r2), v, r1), v, p.e);
  }
}

int check_polynorm(const tlhip_polynorm* p, const char* who);
}  // namespace tlhip
