// Sliding-window attention whose values are its keys: what the decode step (hybrid_step.hip) and the
// prompt-chunk kernel (attn_window.hip) share, and the decode step's block.
//
//   score of the key d places back (d < window): scale t <q_i, k_(i-d)> - d slope
//   out_i = the keys weighted by the softmax of their scores
//
// A key row is loaded once and serves both products.
#pragma once

#include "common.hpp"

namespace tlhip {

constexpr float kLog2e = 1.4426950408889634f;

// v_exp_f32 / v_log_f32 as they are: arguments here never need the library forms' denormal handling
__device__ __forceinline__ float exp2_native(float x) { return __builtin_amdgcn_exp2f(x); }
__device__ __forceinline__ float log2_native(float x) { return __builtin_amdgcn_logf(x); }

// Query multiplier at position p.
__device__ __forceinline__ float query_temperature(int p, float coef, float every) {
  if (every <= 0.f) return 1.f;
  const float steps = (float)floor((double)(p + 1) / (double)every);
  return 1.f + coef * logf(steps + 1.f);
}
// Distance bias per position of head h.
__device__ __forceinline__ float head_slope(int h, int heads, float slope_exp) {
  return slope_exp > 0.f ? exp2f(-slope_exp * (float)(h + 1) / (float)heads) : 0.f;
}
__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }

// all 16 lanes of a DPP row get the row's sum
__device__ __forceinline__ float row16_sum(float v) {
  v += dpp_read<0xB1>(v);    // quad_perm [1,0,3,2]
  v += dpp_read<0x4E>(v);    // quad_perm [2,3,0,1]
  v += dpp_read<0x141>(v);   // row_half_mirror
  v += dpp_read<0x140>(v);   // row_mirror
  return v;
}

// Decode step of the mixer, one block of 512 threads: kv head `kvh`, query heads [h0, h0 + nq) of
// its group (nq <= NQ), split `split` of `S`.
//
// A key row lies across the 16 lanes of a DPP row (NF float4s per lane, 64 columns apart), so a
// wavefront works on four keys at once and a block on 32; each of these 32 streams walks batches
// of four keys with a running (max, sum, output) state per head, and the keys in its registers are
// used for the score and for the output. Batches are dealt round-robin over the streams of all
// splits. The token's own key comes from u, and goes to the ring (block h0 = 0 of split 0); no block
// reads the ring row that is being written.
//
// partials (S > 1): per (head, split) max, sum, then the unnormalised output [ring_ld].
template <int NQ, int NF>
__device__ __forceinline__ void window_step_block(const tlhip_window_attn& a, const float* __restrict__ u,
                                                  float* __restrict__ y, float* __restrict__ partials, int pos,
                                                  int kvh, int h0, int nq, int split, int S, float* smem) {
  constexpr int KB = 4;
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int c = lane & 15, row = lane >> 4;
  const int dim = (int)a.dim, ld = (int)a.ring_ld, heads = (int)a.heads, group = heads / (int)a.kv_heads;
  const int R = (int)a.ring_rows;
  float* qs = smem;                    // [NQ][64 * NF], zeros past dim
  float* ks = smem + NQ * 64 * NF;     // [64 * NF] the new key
  const float temp = query_temperature(pos, a.temp_coef, a.temp_every);
  for (int i = tid; i < (NQ + 1) * 64 * NF; i += 512) {
    const int r = i / (64 * NF), d = i % (64 * NF);
    float v = 0.f;
    if (d < dim) {
      if (r == NQ) v = u[a.k_off + (int64_t)kvh * dim + d];
      else if (r < nq) v = u[a.q_off + (int64_t)(kvh * group + h0 + r) * dim + d] * temp;
    }
    qs[i] = v;
  }
  float* ring = static_cast<float*>(a.ring) + (size_t)kvh * R * ld;
  __syncthreads();
  if (h0 == 0 && split == 0)
    for (int d = tid; d < dim; d += 512) ring[(size_t)(pos % R) * ld + d] = ks[d];
  float4 q[NQ][NF], acc[NQ][NF];
  float m[NQ], l[NQ], sl2[NQ];
  const float sc2 = a.scale * kLog2e;
#pragma unroll
  for (int h = 0; h < NQ; h++) {
    sl2[h] = head_slope(kvh * group + h0 + h, heads, a.slope_exp) * kLog2e;
    m[h] = -INFINITY;
    l[h] = 0.f;
#pragma unroll
    for (int f = 0; f < NF; f++) {
      q[h][f] = *reinterpret_cast<const float4*>(qs + (h * NF + f) * 64 + 4 * c);
      acc[h][f] = make_float4(0.f, 0.f, 0.f, 0.f);
    }
  }
  const auto dot = [&](int h, const float4 (&k)[NF]) {
    float s = 0.f;
#pragma unroll
    for (int f = 0; f < NF; f++)
      s = fmaf(q[h][f].x, k[f].x, fmaf(q[h][f].y, k[f].y, fmaf(q[h][f].z, k[f].z, fmaf(q[h][f].w, k[f].w, s))));
    return row16_sum(s) * sc2;
  };
  if (split == 0 && wave == 0) {       // the token itself (distance 0) starts stream 0's state
    float4 k[NF];
#pragma unroll
    for (int f = 0; f < NF; f++) k[f] = *reinterpret_cast<const float4*>(ks + f * 64 + 4 * c);
#pragma unroll
    for (int h = 0; h < NQ; h++) {
      const float s = dot(h, k);
      if (row == 0) {
        m[h] = s;
        l[h] = 1.f;
#pragma unroll
        for (int f = 0; f < NF; f++) acc[h][f] = k[f];
      }
    }
  }
  const int lo = max(0, pos - (int)a.window + 1), n = pos - lo;    // keys [lo, pos) are in the ring
  const int nb = (n + KB - 1) / KB, streams = 32 * S, sid = split * 32 + wave * 4 + row;
  const auto load = [&](float4 (&k)[KB][NF], int b) {
#pragma unroll
    for (int i = 0; i < KB; i++) {
      const int j = lo + max(min(b * KB + i, n - 1), 0);
      const float* p = ring + (size_t)(j % R) * ld;
#pragma unroll
      for (int f = 0; f < NF; f++) {
        const int d = f * 64 + 4 * c;
        k[i][f] = d < ld ? *reinterpret_cast<const float4*>(p + d) : make_float4(0.f, 0.f, 0.f, 0.f);
      }
    }
  };
  // every lane of the wavefront makes the same number of turns (row sums are exchanged across lanes)
  const int turns = (max(nb - (split * 32 + wave * 4), 0) + streams - 1) / streams;
  float4 k[KB][NF], nx[KB][NF];
  if (turns > 0) load(k, sid);
  for (int t = 0; t < turns; t++) {
    const int b = sid + t * streams;
    if (t + 1 < turns) load(nx, b + streams);
#pragma unroll
    for (int h = 0; h < NQ; h++) {
      float s[KB];
      float mn = m[h];
#pragma unroll
      for (int i = 0; i < KB; i++) {
        const int j = b * KB + i;
        const float d = dot(h, k[i]);
        s[i] = j < n ? d - sl2[h] * (float)(pos - lo - j) : -INFINITY;
        mn = fmaxf(mn, s[i]);
      }
      const float ref = mn == -INFINITY ? 0.f : mn;
      const float corr = exp2_native(m[h] - ref);
      m[h] = mn;
      l[h] *= corr;
#pragma unroll
      for (int f = 0; f < NF; f++) { acc[h][f].x *= corr; acc[h][f].y *= corr; acc[h][f].z *= corr; acc[h][f].w *= corr; }
#pragma unroll
      for (int i = 0; i < KB; i++) {
        const float p = exp2_native(s[i] - ref);
        l[h] += p;
#pragma unroll
        for (int f = 0; f < NF; f++) {
          acc[h][f].x = fmaf(p, k[i][f].x, acc[h][f].x);
          acc[h][f].y = fmaf(p, k[i][f].y, acc[h][f].y);
          acc[h][f].z = fmaf(p, k[i][f].z, acc[h][f].z);
          acc[h][f].w = fmaf(p, k[i][f].w, acc[h][f].w);
        }
      }
    }
#pragma unroll
    for (int i = 0; i < KB; i++)
#pragma unroll
      for (int f = 0; f < NF; f++) k[i][f] = nx[i][f];
  }
  // merge: the four rows of a wavefront by swaps, the wavefronts through LDS
  __syncthreads();                     // qs and ks are done with
  constexpr int WS = 64 * NF + 2;
  float* wl = smem;                    // [8][NQ][max, sum, out[64 * NF]]
#pragma unroll
  for (int h = 0; h < NQ; h++) {
    float M = fmaxf(m[h], __shfl_xor(m[h], 16, kWave));
    M = fmaxf(M, __shfl_xor(M, 32, kWave));
    const float f0 = m[h] == -INFINITY ? 0.f : exp2_native(m[h] - M);
    const auto rows = [&](float v) {
      v *= f0;
      v += __shfl_xor(v, 16, kWave);
      return v + __shfl_xor(v, 32, kWave);
    };
    const float Ls = rows(l[h]);
    float* o = wl + (wave * NQ + h) * WS;
#pragma unroll
    for (int f = 0; f < NF; f++) {
      const float4 v = make_float4(rows(acc[h][f].x), rows(acc[h][f].y), rows(acc[h][f].z), rows(acc[h][f].w));
      if (row == 0) { float* p = o + 2 + f * 64 + 4 * c; p[0] = v.x; p[1] = v.y; p[2] = v.z; p[3] = v.w; }
    }
    if (lane == 0) { o[0] = M; o[1] = Ls; }
  }
  __syncthreads();
  for (int i = tid; i < nq * ld; i += 512) {
    const int h = i / ld, d = i % ld;
    float M = -INFINITY;
#pragma unroll
    for (int w = 0; w < 8; w++) M = fmaxf(M, wl[(w * NQ + h) * WS]);
    float L = 0.f, o = 0.f;
#pragma unroll
    for (int w = 0; w < 8; w++) {
      const float* p = wl + (w * NQ + h) * WS;
      const float f = p[0] == -INFINITY ? 0.f : exp2_native(p[0] - M);
      L = fmaf(f, p[1], L);
      o = fmaf(f, p[2 + d], o);
    }
    const int head = kvh * group + h0 + h;
    if (S == 1) {
      if (d < dim) {
        float v = o / L * a.out_scale;
        if (a.gate_off >= 0) v *= sigmoid_f(u[a.gate_off + (int64_t)head * dim + d]);
        y[a.y_off + (int64_t)head * dim + d] = v;
      }
    } else {
      float* p = partials + ((size_t)head * S + split) * (ld + 2);
      p[2 + d] = o;
      if (d == 0) { p[0] = M; p[1] = L; }
    }
  }
}

// Splits of head `head` -> y. Any block size.
__device__ __forceinline__ void window_merge_head(const tlhip_window_attn& a, const float* __restrict__ u,
                                                  float* __restrict__ y, const float* __restrict__ partials, int head,
                                                  int S) {
  constexpr int U = 8;                                 // splits requested at once
  const int dim = (int)a.dim, ps = (int)a.ring_ld + 2;
  const float* p = partials + (size_t)head * S * ps;
  for (int d = threadIdx.x; d < dim; d += blockDim.x) {
    const float g = a.gate_off >= 0 ? u[a.gate_off + (int64_t)head * dim + d] : 0.f;
    float M = -INFINITY, L = 0.f, o = 0.f;
    for (int s0 = 0; s0 < S; s0 += U) {
      float m[U], l[U], v[U];
#pragma unroll
      for (int k = 0; k < U; k++) {
        const float* q = p + (size_t)min(s0 + k, S - 1) * ps;
        m[k] = q[0];
        l[k] = q[1];
        v[k] = q[2 + d];
      }
#pragma unroll
      for (int k = 0; k < U; k++) {
        if (s0 + k >= S || m[k] == -INFINITY) continue;
        const float n = fmaxf(M, m[k]), fo = exp2_native(M - n), fn = exp2_native(m[k] - n);
        M = n;
        L = L * fo + fn * l[k];
        o = o * fo + fn * v[k];
      }
    }
    float v = o / L * a.out_scale;
    if (a.gate_off >= 0) v *= sigmoid_f(g);
    y[a.y_off + (int64_t)head * dim + d] = v;
  }
}

// What the launchers check of a mixer description (host).
int check_window_attn(const tlhip_window_attn* a, const char* who);
}  // namespace tlhip
