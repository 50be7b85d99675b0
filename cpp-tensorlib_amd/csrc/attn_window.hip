// Prompt chunks of the sliding-window attention whose values are its keys, in two forms, and the copy of
// a chunk's keys into the ring.
//
// window_chunk_kernel, the exact form, runs on the fp32 matrix pipe. A block owns one query head and 32 consecutive positions; its NW wavefronts deal the 32-key tiles
// that the window touches, each with its own running (max, sum, output) state, merged through LDS at
// the end. v_mfma_f32_32x32x2_f32 multiplies f32 by f32 exactly. Both products are formed transposed:
//   S^T = K Q^T : lane (l % 32) holds 16 scores of query l % 32, keys 8a + 4 (l / 32) + b in
//                 register 4a + b;
//   O^T = K^T P^T : such a register is, as it stands, the P operand of the step that adds keys
//                 8a + b and 8a + 4 + b.
// So probabilities need no exchange, a query's maximum and sum are in-lane reductions and one swap of
// the two halves, and the softmax correction is one number per lane. The key tile sits in LDS once and
// is the operand of both products (rows for the first, columns for the second).
// Tiles start at multiples of 32 positions, and the ring holds a multiple of 32 rows: a tile never
// wraps inside the ring.
//
// window_terms_kernel runs on the 16-bit matrix cores: every f32 operand is cut into two bf16 terms, each
// rounded to nearest (16 significant bits, f32's range), and a product is formed from the three term
// pairs that hold a first term, fp32 sums. Scores, softmax and sums stay f32. A block owns one kv head:
// its eight wavefronts are the query heads of the group (and, for small groups, consecutive runs of 32
// positions) and share one 32-key tile, which all 512 threads cut into terms while the tile before it is
// worked on: rows for K Q^T, and keys in the order in which the score registers hold them, as the
// operand of K^T P^T. Tiles are dealt over S blocks so that the chip is filled; window_join_kernel
// adds those up.
#include "attn_window.hpp"

#include <algorithm>

namespace tlhip {

typedef float f32x16 __attribute__((ext_vector_type(16)));
typedef float f32x4 __attribute__((ext_vector_type(4)));

template <int D, int NW>
struct WindowLds {
  static constexpr int KS = D + 4;
  static constexpr int kRegion = 32 * KS;                 // floats: Q, and one key tile per wavefront
  static constexpr size_t kBytes = (size_t)((1 + NW) * kRegion + NW * 64) * sizeof(float);
};

// The 32 key rows of a tile into registers, 16 bytes per lane and load; rows at or past kend are clamped
// to the last one (masked when used).
template <int D>
__device__ __forceinline__ void window_tile(f32x4 (&k)[D / 8], const float* __restrict__ ring, int tile, int kend, int R,
                                            int lane) {
  const float* base = ring + (size_t)((tile * 32) % R) * D;
  const int last = kend - 1 - tile * 32;
#pragma unroll
  for (int i = 0; i < D / 8; i++) {
    const int slot = lane + 64 * i, key = slot / (D / 4), c4 = slot % (D / 4);
    k[i] = *reinterpret_cast<const f32x4*>(base + (size_t)min(key, last) * D + 4 * c4);
  }
}

template <int D, int NW>
__global__ __launch_bounds__(64 * NW, 1) void window_chunk_kernel(const float* __restrict__ u, int64_t ldu,
                                                                 float* __restrict__ y, int64_t ldy,
                                                                 const tlhip_window_attn a, int T, int pos0) {
  using L = WindowLds<D, NW>;
  constexpr int KS = L::KS, NT = 64 * NW;
  constexpr int kLoads = D / 8;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int l31 = lane & 31, hi = lane >> 5;
  const int h = blockIdx.x, dim = (int)a.dim, heads = (int)a.heads, window = (int)a.window;
  const int p0 = (int)(gridDim.y - 1 - blockIdx.y) * 32;
  const int R = (int)a.ring_rows;
  const float* ring = static_cast<const float*>(a.ring) + (size_t)(h / (heads / (int)a.kv_heads)) * R * D;
  float* Qs = lds;
  float* K = lds + (1 + wave) * L::kRegion;
  float* stat = lds + (1 + NW) * L::kRegion;              // [NW][max 32 | sum 32]
  const int kend = min(pos0 + p0 + 32, pos0 + T);         // keys of this block end here
  const int kt0 = max(0, pos0 + p0 - window + 1) >> 5, kt1 = (kend + 31) >> 5;

  for (int r = wave; r < 32; r += NW) {      // queries times their temperature (rows beyond T clamped, never stored)
    const int t = min(p0 + r, T - 1);
    const float temp = query_temperature(pos0 + t, a.temp_coef, a.temp_every);
    const float* q = u + (size_t)t * ldu + a.q_off + (size_t)h * dim;
    for (int d = lane; d < D; d += 64) Qs[r * KS + d] = d < dim ? q[d] * temp : 0.f;
  }

  f32x4 kreg[kLoads];
  window_tile<D>(kreg, ring, min(kt0 + wave, kt1 - 1), kend, R, lane);
  __syncthreads();

  f32x16 o[D / 32];
#pragma unroll
  for (int dt = 0; dt < D / 32; dt++)
#pragma unroll
    for (int v = 0; v < 16; v++) o[dt][v] = 0.f;
  float m = -INFINITY, lsum = 0.f;
  const int qpos = pos0 + p0 + l31;
  const float sc2 = a.scale * kLog2e, sl2 = head_slope(h, heads, a.slope_exp) * kLog2e;
  for (int kt = kt0 + wave; kt < kt1; kt += NW) {
#pragma unroll
    for (int i = 0; i < kLoads; i++) {
      const int slot = lane + 64 * i, key = slot / (D / 4), c4 = slot % (D / 4);
      *reinterpret_cast<f32x4*>(K + key * KS + 4 * c4) = kreg[i];
    }
    window_tile<D>(kreg, ring, min(kt + NW, kt1 - 1), kend, R, lane);
    f32x16 s;
#pragma unroll
    for (int v = 0; v < 16; v++) s[v] = 0.f;
#pragma unroll
    for (int g = 0; g < D / 8; g++) {
      const float4 qf = *reinterpret_cast<const float4*>(Qs + l31 * KS + 8 * g + 4 * hi);
      const float4 kf = *reinterpret_cast<const float4*>(K + l31 * KS + 8 * g + 4 * hi);
      s = __builtin_amdgcn_mfma_f32_32x32x2f32(kf.x, qf.x, s, 0, 0, 0);
      s = __builtin_amdgcn_mfma_f32_32x32x2f32(kf.y, qf.y, s, 0, 0, 0);
      s = __builtin_amdgcn_mfma_f32_32x32x2f32(kf.z, qf.z, s, 0, 0, 0);
      s = __builtin_amdgcn_mfma_f32_32x32x2f32(kf.w, qf.w, s, 0, 0, 0);
    }
    const int dist0 = qpos - kt * 32 - 4 * hi;            // distance to key 8a + b of this lane: dist0 - (8a + b)
    float mx = m;
#pragma unroll
    for (int v = 0; v < 16; v++) {
      const int dist = dist0 - (8 * (v >> 2) + (v & 3));
      s[v] = dist >= 0 && dist < window ? s[v] * sc2 - sl2 * (float)dist : -INFINITY;
      mx = fmaxf(mx, s[v]);
    }
    const LanePair mp = swap32(mx, mx);
    mx = fmaxf(mp.first, mp.second);
    const float ref = mx == -INFINITY ? 0.f : mx;
    const float corr = exp2_native(m - ref);
    m = mx;
    float ps = 0.f;
#pragma unroll
    for (int v = 0; v < 16; v++) {
      s[v] = exp2_native(s[v] - ref);
      ps += s[v];
    }
    lsum = lsum * corr + ps;                              // this half's keys; the halves meet at the end
#pragma unroll
    for (int dt = 0; dt < D / 32; dt++)
#pragma unroll
      for (int v = 0; v < 16; v++) o[dt][v] *= corr;
#pragma unroll
    for (int v = 0; v < 16; v++) {
      const float* kp = K + (8 * (v >> 2) + 4 * hi + (v & 3)) * KS + l31;
#pragma unroll
      for (int dt = 0; dt < D / 32; dt++) o[dt] = __builtin_amdgcn_mfma_f32_32x32x2f32(kp[dt * 32], s[v], o[dt], 0, 0, 0);
    }
  }
  // merge: each wavefront leaves O [32][D], max and sum; every row is then finished by NT / 32 threads
#pragma unroll
  for (int dt = 0; dt < D / 32; dt++)
#pragma unroll
    for (int q = 0; q < 4; q++)
      *reinterpret_cast<float4*>(K + l31 * KS + dt * 32 + 8 * q + 4 * hi) =
          make_float4(o[dt][4 * q], o[dt][4 * q + 1], o[dt][4 * q + 2], o[dt][4 * q + 3]);
  const LanePair lp = swap32(lsum, lsum);
  if (hi == 0) { stat[wave * 64 + l31] = m; stat[wave * 64 + 32 + l31] = lp.first + lp.second; }
  __syncthreads();
  constexpr int TPR = NT / 32;
  const int row = tid / TPR, t = p0 + row;
  if (t >= T) return;
  float f[NW], M = -INFINITY, Ls = 0.f;
#pragma unroll
  for (int w = 0; w < NW; w++) M = fmaxf(M, stat[w * 64 + row]);
#pragma unroll
  for (int w = 0; w < NW; w++) {
    const float mw = stat[w * 64 + row];
    f[w] = mw == -INFINITY ? 0.f : exp2_native(mw - M);
    Ls = fmaf(f[w], stat[w * 64 + 32 + row], Ls);
  }
  const float inv = a.out_scale / Ls;
  const float* up = u + (size_t)t * ldu + a.gate_off + (size_t)h * dim;
  float* yp = y + (size_t)t * ldy + a.y_off + (size_t)h * dim;
  for (int d = tid % TPR; d < dim; d += TPR) {
    float v = 0.f;
#pragma unroll
    for (int w = 0; w < NW; w++) v = fmaf(f[w], lds[(1 + w) * L::kRegion + row * KS + d], v);
    v *= inv;
    if (a.gate_off >= 0) v *= sigmoid_f(up[d]);
    yp[d] = v;
  }
}

// ---- two bf16 terms ------------------------------------------------------------------------------
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef uint32_t u32x2 __attribute__((ext_vector_type(2)));
typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
typedef float f32x2 __attribute__((ext_vector_type(2)));

// two f32 rounded to bf16 (nearest even): x0 in the low half. One v_cvt_pk_bf16_f32, left to the compiler:
// it knows what must stand between a transcendental instruction and a reader of its result.
typedef __bf16 bf16x2 __attribute__((ext_vector_type(2)));
__device__ __forceinline__ uint32_t bf16_pair(float x0, float x1) {
  return __builtin_bit_cast(uint32_t, __builtin_convertvector(f32x2{x0, x1}, bf16x2));
}
__device__ __forceinline__ void two_terms(float x0, float x1, uint32_t& first, uint32_t& second) {
  first = bf16_pair(x0, x1);
  second = bf16_pair(x0 - bf16_lo(first), x1 - bf16_hi(first));
}
__device__ __forceinline__ bf16x8 as_bf16x8(u32x4 v) { return __builtin_bit_cast(bf16x8, v); }
__device__ __forceinline__ f32x16 mfma_bf16(bf16x8 a, bf16x8 b, f32x16 c) {
  return __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, b, c, 0, 0, 0);
}

struct TermPlan {
  int gh;        // query heads of a block
  int subs;      // blocks that share a kv head's group
  int pt;        // runs of 32 positions of a block
  int S;         // key splits
};

// LDS: two buffers, each K [term][32 keys][D + 8] and KT [term][key step 2][half 2][D][8 keys], bf16.
template <int D>
struct TermLds {
  static constexpr int kKRow = D + 8, kK = 32 * kKRow, kT = 4 * D * 8;
  static constexpr int kBuf = 2 * kK + 2 * kT;              // bf16 elements of one buffer
  static constexpr size_t kBytes = (size_t)2 * kBuf * 2;
};

template <int D>
__global__ __launch_bounds__(512, 1) void window_terms_kernel(const float* __restrict__ u, int64_t ldu, float* __restrict__ y,
                                                             int64_t ldy, const tlhip_window_attn a, int T, int pos0,
                                                             const TermPlan plan, float* __restrict__ acc_out,
                                                             float* __restrict__ stat_out) {
  using L = TermLds<D>;
  extern __shared__ __attribute__((aligned(16))) uint16_t bl[];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int l31 = lane & 31, hi = lane >> 5;
  const int heads = (int)a.heads, group = heads / (int)a.kv_heads, dim = (int)a.dim, window = (int)a.window, R = (int)a.ring_rows;
  const int kvh = blockIdx.x / plan.subs, sub = blockIdx.x % plan.subs;
  const int hh = sub * plan.gh + wave % plan.gh, run = wave / plan.gh, h = kvh * group + hh;
  const int b0 = (int)(gridDim.y - 1 - blockIdx.y) * 32 * plan.pt, p0 = b0 + 32 * run;
  const bool works = hh < group && run < plan.pt && p0 < T;
  const float* ring = static_cast<const float*>(a.ring) + (size_t)kvh * R * D;
  const int kend = min(pos0 + b0 + 32 * plan.pt, pos0 + T);
  const int kt0 = max(0, pos0 + b0 - window + 1) >> 5, kt1 = (kend + 31) >> 5;
  // the tiles this wavefront's 32 queries see
  const int wt0 = works ? max(0, pos0 + p0 - window + 1) >> 5 : 0, wt1 = works ? (min(pos0 + p0 + 32, pos0 + T) + 31) >> 5 : 0;

  // staging: a thread cuts two columns of four keys
  constexpr int kTasks = 8 * (D / 2);
  const int kq = tid / (D / 2), d2 = 2 * (tid % (D / 2));
  const bool stages = tid < kTasks;
  f32x2 kreg[4];
  const auto request = [&](f32x2 (&k)[4], int tile, int first_row) {
    const float* base = ring + (size_t)first_row * D + d2;
    const int last = kend - 1 - tile * 32;
#pragma unroll
    for (int i = 0; i < 4; i++) k[i] = *reinterpret_cast<const f32x2*>(base + (size_t)min(4 * kq + i, last) * D);
  };
  const auto stage = [&](const f32x2 (&k)[4], int buf) {
    uint16_t *K = bl + buf * L::kBuf, *KT = K + 2 * L::kK;
    uint32_t t0[4], t1[4];             // of each key: both columns' first and second terms
#pragma unroll
    for (int i = 0; i < 4; i++) {
      two_terms(k[i][0], k[i][1], t0[i], t1[i]);
      *reinterpret_cast<uint32_t*>(K + (4 * kq + i) * L::kKRow + d2) = t0[i];
      *reinterpret_cast<uint32_t*>(K + L::kK + (4 * kq + i) * L::kKRow + d2) = t1[i];
    }
    // keys 4kq .. 4kq + 3 are elements 4 (kq / 2 % 2) .. of key step kq / 4, lane half kq % 2
    const int unit = ((kq >> 2) * 2 + (kq & 1)) * D + d2, off = 4 * ((kq >> 1) & 1);
    const auto column = [](const uint32_t (&t)[4], uint32_t pick) {
      return u32x2{__builtin_amdgcn_perm(t[1], t[0], pick), __builtin_amdgcn_perm(t[3], t[2], pick)};
    };
#pragma unroll
    for (int c = 0; c < 2; c++) {
      const uint32_t pick = c ? 0x07060302u : 0x05040100u;   // the high or low halves of two words
      *reinterpret_cast<u32x2*>(KT + (unit + c) * 8 + off) = column(t0, pick);
      *reinterpret_cast<u32x2*>(KT + L::kT + (unit + c) * 8 + off) = column(t1, pick);
    }
  };
  // newest keys first: the distance bias makes them the likely maxima, which then seldom move
  int kt = kt1 - 1 - (int)blockIdx.z;
  int row = kt >= kt0 ? (kt * 32) % R : 0;             // of tile kt in the ring; a step back is 32 S rows
  const int back = (32 * plan.S) % R;
  if (stages && kt >= kt0) request(kreg, kt, row);

  // queries times their temperature, cut into terms: lane (hi, l31) holds columns 16s + 8hi .. + 7 of query l31
  bf16x8 q0[D / 16], q1[D / 16];
  {
    const int t = min(p0 + l31, T - 1);
    const float temp = query_temperature(pos0 + t, a.temp_coef, a.temp_every);
    const int64_t qo = a.q_off + (int64_t)min(h, heads - 1) * dim;
    const float* q = u + (size_t)t * ldu + qo;
    f32x4 x[D / 8];
    // (uniform: every row of queries starts on 16 bytes and holds whole quads)
    if (((reinterpret_cast<uintptr_t>(u) & 15) | ((qo | ldu | dim) & 3)) == 0) {
#pragma unroll
      for (int i = 0; i < D / 8; i++) x[i] = *reinterpret_cast<const f32x4*>(q + min(16 * (i >> 1) + 8 * hi + 4 * (i & 1), dim - 4));
    } else {
#pragma unroll
      for (int i = 0; i < D / 8; i++)
#pragma unroll
        for (int j = 0; j < 4; j++) x[i][j] = q[min(16 * (i >> 1) + 8 * hi + 4 * (i & 1) + j, dim - 1)];
    }
#pragma unroll
    for (int s = 0; s < D / 16; s++) {
      u32x4 f, g;
#pragma unroll
      for (int j = 0; j < 4; j++) {
        const int d = 16 * s + 8 * hi + 2 * j;
        const f32x4 v = x[2 * s + (j >> 1)];
        uint32_t f1, g1;
        two_terms(d < dim ? v[2 * (j & 1)] * temp : 0.f, d + 1 < dim ? v[2 * (j & 1) + 1] * temp : 0.f, f1, g1);
        f[j] = f1;
        g[j] = g1;
      }
      q0[s] = as_bf16x8(f);
      q1[s] = as_bf16x8(g);
    }
  }
  f32x16 o[D / 32];
#pragma unroll
  for (int dt = 0; dt < D / 32; dt++)
#pragma unroll
    for (int v = 0; v < 16; v++) o[dt][v] = 0.f;
  float m = -INFINITY, lsum = 0.f;
  const int qpos = pos0 + p0 + l31;
  const float sc2 = a.scale * kLog2e, sl2 = head_slope(h, heads, a.slope_exp) * kLog2e;

  const auto step_back = [&] {
    row -= back;
    if (row < 0) row += R;
  };
  if (stages && kt >= kt0) stage(kreg, 0);
  step_back();
  if (stages && kt - plan.S >= kt0) request(kreg, kt - plan.S, row);
  __syncthreads();
  for (int buf = 0; kt >= kt0; kt -= plan.S, buf ^= 1) {
    if (kt >= wt0 && kt < wt1) {
      const uint16_t *K = bl + buf * L::kBuf, *KT = K + 2 * L::kK;
      f32x16 s, r;                     // first x first, and the two mixed pairs
#pragma unroll
      for (int v = 0; v < 16; v++) { s[v] = 0.f; r[v] = 0.f; }
#pragma unroll
      for (int g = 0; g < D / 16; g++) {
        const bf16x8 k0 = *reinterpret_cast<const bf16x8*>(K + l31 * L::kKRow + 16 * g + 8 * hi);
        const bf16x8 k1 = *reinterpret_cast<const bf16x8*>(K + L::kK + l31 * L::kKRow + 16 * g + 8 * hi);
        s = mfma_bf16(k0, q0[g], s);
        r = mfma_bf16(k0, q1[g], r);
        r = mfma_bf16(k1, q0[g], r);
      }
      const int dist0 = qpos - kt * 32 - 4 * hi;
      float mx = m;
#pragma unroll
      for (int v = 0; v < 16; v++) {
        const int dist = dist0 - (8 * (v >> 2) + (v & 3));
        s[v] = dist >= 0 && dist < window ? (s[v] + r[v]) * sc2 - sl2 * (float)dist : -INFINITY;
        mx = fmaxf(mx, s[v]);
      }
      const LanePair mp = swap32(mx, mx);
      mx = fmaxf(mp.first, mp.second);
      const float ref = mx == -INFINITY ? 0.f : mx;
      if (__builtin_amdgcn_ballot_w64(mx > m)) {       // some query's maximum moved
        const float corr = exp2_native(m - ref);
        m = mx;
        lsum *= corr;
#pragma unroll
        for (int dt = 0; dt < D / 32; dt++)
#pragma unroll
          for (int v = 0; v < 16; v++) o[dt][v] *= corr;
      }
      u32x4 w0[2], w1[2];
      float ps = 0.f;
#pragma unroll
      for (int v = 0; v < 16; v += 2) {
        const float pa = exp2_native(s[v] - ref), pb = exp2_native(s[v + 1] - ref);
        ps += pa + pb;
        uint32_t f, g;
        two_terms(pa, pb, f, g);
        w0[v >> 3][(v & 7) >> 1] = f;
        w1[v >> 3][(v & 7) >> 1] = g;
      }
      lsum += ps;
#pragma unroll
      for (int st = 0; st < 2; st++)
#pragma unroll
        for (int dt = 0; dt < D / 32; dt++) {
          const uint16_t* p = KT + ((st * 2 + hi) * D + dt * 32 + l31) * 8;
          const bf16x8 v0 = *reinterpret_cast<const bf16x8*>(p);
          const bf16x8 v1 = *reinterpret_cast<const bf16x8*>(p + L::kT);
          o[dt] = mfma_bf16(v1, as_bf16x8(w0[st]), o[dt]);
          o[dt] = mfma_bf16(v0, as_bf16x8(w1[st]), o[dt]);
          o[dt] = mfma_bf16(v0, as_bf16x8(w0[st]), o[dt]);
        }
    }
    // the next tile into the other buffer (last read before the barrier that ended the turn before)
    if (stages && kt - plan.S >= kt0) stage(kreg, buf ^ 1);
    step_back();
    if (stages && kt - 2 * plan.S >= kt0) request(kreg, kt - 2 * plan.S, row);
    __syncthreads();
  }
  const int t = p0 + l31;
  const LanePair lp = swap32(lsum, lsum);
  const float Ls = lp.first + lp.second;
  if (!works || t >= T) return;
  if (plan.S > 1) {
    const size_t row = ((size_t)blockIdx.z * T + t) * heads + h;
    if (hi == 0) { stat_out[2 * row] = m; stat_out[2 * row + 1] = Ls; }
#pragma unroll
    for (int dt = 0; dt < D / 32; dt++)
#pragma unroll
      for (int q = 0; q < 4; q++)
        *reinterpret_cast<float4*>(acc_out + row * D + dt * 32 + 8 * q + 4 * hi) =
            make_float4(o[dt][4 * q], o[dt][4 * q + 1], o[dt][4 * q + 2], o[dt][4 * q + 3]);
    return;
  }
  const float inv = a.out_scale / Ls;
  if (a.gate_off >= 0) {
    const float* gp = u + (size_t)t * ldu + a.gate_off + (size_t)h * dim;
#pragma unroll
    for (int dt = 0; dt < D / 32; dt++) {
      float g[16];
#pragma unroll
      for (int v = 0; v < 16; v++) g[v] = gp[min(dt * 32 + 8 * (v >> 2) + 4 * hi + (v & 3), dim - 1)];
#pragma unroll
      for (int v = 0; v < 16; v++) o[dt][v] *= sigmoid_f(g[v]);
    }
  }
  float* yp = y + (size_t)t * ldy + a.y_off + (size_t)h * dim;
#pragma unroll
  for (int dt = 0; dt < D / 32; dt++)
#pragma unroll
    for (int v = 0; v < 16; v++) {
      const int d = dt * 32 + 8 * (v >> 2) + 4 * hi + (v & 3);
      if (d < dim) yp[d] = o[dt][v] * inv;
    }
}

// The key splits of (token, head) rows -> y, D / 4 lanes to a row. `i` numbers threads.
template <int D>
__device__ __forceinline__ void window_join(const float* __restrict__ u, int64_t ldu, float* __restrict__ y, int64_t ldy,
                                            const tlhip_window_attn& a, int T, int S, const float* __restrict__ acc,
                                            const float* __restrict__ stat, size_t i) {
  constexpr int LR = D / 4, U = 4;                // splits requested at once
  const int heads = (int)a.heads, dim = (int)a.dim;
  const size_t rows = (size_t)T * heads, r = i / LR;
  const int d = 4 * (int)(i % LR);
  if (r >= rows || d >= dim) return;
  const int t = (int)(r / heads), h = (int)(r % heads);
  const float* gp = u + (size_t)t * ldu + a.gate_off + (size_t)h * dim + d;
  const bool gated = a.gate_off >= 0;
  float g[4];
#pragma unroll
  for (int j = 0; j < 4; j++) g[j] = gated && d + j < dim ? gp[j] : 0.f;
  float M = -INFINITY, Ls = 0.f;
  f32x4 o = {0.f, 0.f, 0.f, 0.f};
  for (int s0 = 0; s0 < S; s0 += U) {
    f32x4 v[U];
    f32x2 st[U];
#pragma unroll
    for (int k = 0; k < U; k++) {
      const size_t at = (size_t)min(s0 + k, S - 1) * rows + r;
      v[k] = *reinterpret_cast<const f32x4*>(acc + at * D + d);
      st[k] = *reinterpret_cast<const f32x2*>(stat + 2 * at);
    }
#pragma unroll
    for (int k = 0; k < U; k++) {
      if (s0 + k >= S || st[k][0] == -INFINITY) continue;
      const float m = fmaxf(M, st[k][0]), fo = exp2_native(M - m), fn = exp2_native(st[k][0] - m);
      M = m;
      Ls = Ls * fo + fn * st[k][1];
#pragma unroll
      for (int j = 0; j < 4; j++) o[j] = o[j] * fo + fn * v[k][j];
    }
  }
  const float inv = a.out_scale / Ls;
  float* yp = y + (size_t)t * ldy + a.y_off + (size_t)h * dim + d;
#pragma unroll
  for (int j = 0; j < 4; j++)
    if (d + j < dim) yp[j] = o[j] * inv * (gated ? sigmoid_f(g[j]) : 1.f);
}

template <int D>
__global__ __launch_bounds__(256) void window_join_kernel(const float* __restrict__ u, int64_t ldu, float* __restrict__ y,
                                                          int64_t ldy, const tlhip_window_attn a, int T, int S,
                                                          const float* __restrict__ acc, const float* __restrict__ stat) {
  window_join<D>(u, ldu, y, ldy, a, T, S, acc, stat, (size_t)blockIdx.x * 256 + threadIdx.x);
}

template <int D>
static int launch_terms(const float* u, int64_t ldu, float* y, int64_t ldy, const tlhip_window_attn& a, int T, int pos0) {
  Context& c = ctx();
  const int group = (int)(a.heads / a.kv_heads);
  TermPlan p{};
  p.gh = group < 8 ? group : 8;
  p.subs = (group + p.gh - 1) / p.gh;
  p.pt = 8 / p.gh;
  while (p.pt > 1 && 32 * (p.pt - 1) >= T) p.pt--;
  const int runs = (T + 32 * p.pt - 1) / (32 * p.pt);
  const int64_t blocks = a.kv_heads * p.subs * runs, tiles = (std::min<int64_t>(a.window, pos0 + T) + 32 * p.pt + 31) / 32;
  p.S = (int)std::max<int64_t>(1, std::min<int64_t>({c.cus / blocks, tiles / 3, 16}));
  float *acc = nullptr, *stat = nullptr;
  if (p.S > 1) {
    const size_t rows = (size_t)p.S * T * a.heads;
    acc = static_cast<float*>(scratch(rows * (D + 2) * sizeof(float)));   // rows of D are 16-byte aligned, then the pairs
    if (!acc) return fail(TLHIP_ENOMEM, "tlhip_window_attn_chunk: no scratch");
    stat = acc + rows * D;
  }
  auto fn = window_terms_kernel<D>;
  const size_t lds = TermLds<D>::kBytes;
  const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(fn), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
  if (e != hipSuccess) return hip_fail(e, "hipFuncSetAttribute(LDS)");
  hipLaunchKernelGGL(fn, dim3((unsigned)(a.kv_heads * p.subs), (unsigned)runs, (unsigned)p.S), dim3(512), lds, c.stream, u, ldu, y, ldy,
                     a, T, pos0, p, acc, stat);
  if (p.S > 1)
    hipLaunchKernelGGL(window_join_kernel<D>, dim3((unsigned)(((size_t)T * a.heads * (D / 4) + 255) / 256)), dim3(256), 0, c.stream, u, ldu, y,
                       ldy, a, T, p.S, acc, stat);
  TLHIP_CHECK_LAUNCH(TLHIP_C_WINDOW_ATTN);
}

// Keys of the chunk's tokens -> ring rows, zeros past dim.
__global__ __launch_bounds__(256) void window_fill_kernel(const float* __restrict__ u, int64_t ldu, const tlhip_window_attn a,
                                                          int T, int pos0) {
  const int ld = (int)a.ring_ld, dim = (int)a.dim, kvh = (int)a.kv_heads;
  const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= (size_t)T * kvh * ld) return;
  const int d = (int)(i % ld), g = (int)(i / ld % kvh), t = (int)(i / ld / kvh);
  static_cast<float*>(a.ring)[((size_t)g * a.ring_rows + (pos0 + t) % a.ring_rows) * ld + d] =
      d < dim ? u[(size_t)t * ldu + a.k_off + (size_t)g * dim + d] : 0.f;
}

template <int D, int NW>
static int launch_window(const float* u, int64_t ldu, float* y, int64_t ldy, const tlhip_window_attn& a, int T, int pos0) {
  Context& c = ctx();
  auto fn = window_chunk_kernel<D, NW>;
  const int lds = (int)WindowLds<D, NW>::kBytes;
  if (lds > c.lds_per_cu) return fail(TLHIP_EUNSUPPORTED, "tlhip_window_attn_chunk: not enough LDS");
  const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(fn), hipFuncAttributeMaxDynamicSharedMemorySize, lds);
  if (e != hipSuccess) return hip_fail(e, "hipFuncSetAttribute(LDS)");
  hipLaunchKernelGGL(fn, dim3((unsigned)a.heads, (unsigned)((T + 31) / 32)), dim3(64 * NW), (size_t)lds, c.stream, u, ldu, y, ldy,
                     a, T, pos0);
  TLHIP_CHECK_LAUNCH(TLHIP_C_WINDOW_ATTN);
}

static int check_chunk(const void* u, int64_t ldu, int64_t T, int64_t pos0, const tlhip_window_attn* a, const char* who) {
  if (!u || !a || ldu <= 0) return fail(TLHIP_EINVAL, "%s: bad operands", who);
  if (T <= 0 || T > (1 << 20) || pos0 < 0 || pos0 + T > (1 << 30)) return fail(TLHIP_EINVAL, "%s: bad chunk", who);
  if (int rc = check_window_attn(a, who)) return rc;
  if (T + a->window - 1 > a->ring_rows && pos0 + T > a->ring_rows)
    return fail(TLHIP_EINVAL, "%s: the key ring does not hold the window and the chunk", who);
  return TLHIP_OK;
}

}  // namespace tlhip

using namespace tlhip;

extern "C" {

int tlhip_window_fill(const void* u, int64_t ldu, const tlhip_window_attn* at, int64_t T, int64_t pos0) {
  TLHIP_REQUIRE_READY();
  if (int rc = check_chunk(u, ldu, T, pos0, at, "tlhip_window_fill")) return rc;
  const size_t n = (size_t)T * at->kv_heads * at->ring_ld;
  window_fill_kernel<<<dim3((unsigned)((n + 255) / 256)), dim3(256), 0, ctx().stream>>>(static_cast<const float*>(u), ldu, *at,
                                                                                   (int)T, (int)pos0);
  TLHIP_CHECK_LAUNCH(TLHIP_C_KV_FILL);
}

int tlhip_window_attn_chunk(const void* u, int64_t ldu, void* y, int64_t ldy, const tlhip_window_attn* at, int64_t T,
                            int64_t pos0, int exact) {
  TLHIP_REQUIRE_READY();
  if (!y || ldy <= 0) return fail(TLHIP_EINVAL, "tlhip_window_attn_chunk: bad operands");
  if (int rc = check_chunk(u, ldu, T, pos0, at, "tlhip_window_attn_chunk")) return rc;
  const float* pu = static_cast<const float*>(u);
  float* py = static_cast<float*>(y);
  if (!exact && T >= 16) switch (at->ring_ld) {
      case 32: return launch_terms<32>(pu, ldu, py, ldy, *at, (int)T, (int)pos0);
      case 64: return launch_terms<64>(pu, ldu, py, ldy, *at, (int)T, (int)pos0);
      case 96: return launch_terms<96>(pu, ldu, py, ldy, *at, (int)T, (int)pos0);
      case 128: return launch_terms<128>(pu, ldu, py, ldy, *at, (int)T, (int)pos0);
      default: break;                // larger heads: the exact form
    }
  // few key tiles: more wavefronts than tiles would only add to the merge
  const bool few = at->window <= 96;
#define TLHIP_WIN(D, NW) return launch_window<D, NW>(pu, ldu, py, ldy, *at, (int)T, (int)pos0)
  switch (at->ring_ld) {
    case 32: if (few) TLHIP_WIN(32, 4); else TLHIP_WIN(32, 8);
    case 64: if (few) TLHIP_WIN(64, 4); else TLHIP_WIN(64, 8);
    case 96: if (few) TLHIP_WIN(96, 4); else TLHIP_WIN(96, 8);
    case 128: if (few) TLHIP_WIN(128, 4); else TLHIP_WIN(128, 8);
    case 192: TLHIP_WIN(192, 4);
    case 256: TLHIP_WIN(256, 3);
    default: return fail(TLHIP_EUNSUPPORTED, "tlhip_window_attn_chunk: no kernel for this head size");
  }
#undef TLHIP_WIN
}

}  // extern "C"
