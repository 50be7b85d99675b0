// Latent attention: keys and values of all heads are linear images of one cached latent per position,
//   k_h = [uk_h c | r],  v_h = uv_h c,   c: L numbers (RMS-normed), r: R rotated numbers shared by all heads.
// The up-projections are moved to the query's side and behind the sum,
//   q_h . k_h = (uk_h^T qn_h) . c + qr_h . r,     sum_j p_j v_hj = uv_h (sum_j p_j c_j),
// so all heads of all tokens read the same cache row [c | r]: attention with ONE key head of L + R dims whose
// values are the first L of them. Query rows (token, head) are packed 32 to a tile, 32 heads of one token or
// a few heads of several, and every cached byte is read once per tile.
//
// Cache. Two copies, each in the register image of the matrix-core operand it becomes, so that no kernel
// transposes anything: per tile of 32 keys
//   keys    [plane][DS dim steps of 16][lane][8]     lane (g, c): key c, dims 16 s + 8 g ..
//   values  [plane][LT tiles of 32 dims][2 key steps][lane][8]    lane (g, c): dim 32 t + c, keys wide_key(u, g, j)
// A value is kept as NC bf16 terms (planes): one rounded to nearest, or three that add up to the f32 exactly.
// Products run on v_mfma_f32_32x32x16_bf16 with queries and probabilities in NQ terms of their own (two or
// three), every pair of terms multiplied; scores, softmax and sums are f32. Both products are transposed
// (S^T = K Q^T, O^T = V^T P^T): a lane owns one query row, and the scores' registers are the second
// product's operand as they are.
//
// Launches: queries into operand images and new cache rows (latent_query_kernel; in prompt chunks of the one-plane
// form latent_query_mfma_kernel), attention (latent_attend_kernel, three planes: latent_attend_exact_kernel; blocks:
// query tile x key split), splits joined, uv, gate (latent_out_kernel; latent_out_mfma_kernel).
#include "common.hpp"

#include <algorithm>

namespace tlhip {
namespace latent {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x16 __attribute__((ext_vector_type(16)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
typedef uint32_t u32x2 __attribute__((ext_vector_type(2)));

struct Dims {
  int H, D, R, V, L, DS, LT, NC;
};
__host__ __device__ inline Dims dims_of(const tlhip_latent_attn& a) {
  Dims d;
  d.H = (int)a.heads; d.D = (int)a.dim; d.R = (int)a.rot_dim; d.V = (int)a.vdim; d.L = (int)a.kv_rank;
  d.DS = (d.L + d.R + 15) / 16;
  d.LT = (d.L + 31) / 32;
  d.NC = (int)a.planes;
  return d;
}
__host__ __device__ inline int up8(int n) { return (n + 7) & ~7; }

// x in N bf16 terms, the first N - 1 by truncation when N is 3 (the sum is exact), else rounded to nearest
template <int N>
__device__ __forceinline__ void cut(float x, uint16_t (&t)[N]) {
  if constexpr (N == 3) {
    const uint32_t h = __float_as_uint(x) & 0xffff0000u;
    const float r1 = x - __uint_as_float(h);
    const uint32_t m = __float_as_uint(r1) & 0xffff0000u;
    t[0] = (uint16_t)(h >> 16);
    t[1] = (uint16_t)(m >> 16);
    t[2] = (uint16_t)(__float_as_uint(r1 - __uint_as_float(m)) >> 16);
  } else {
    float r = x;
#pragma unroll
    for (int i = 0; i < N; i++) {
      t[i] = f32_to_bf16_rne(r);
      r -= __uint_as_float((uint32_t)t[i] << 16);
    }
  }
}

// where dim e of key row p lies in the key image, dim e in the value image (elements, plane 0)
__device__ __forceinline__ size_t key_at(const Dims& d, int p, int e) {
  return ((size_t)(p >> 5) * d.NC * d.DS + (e >> 4)) * 512 + (((e >> 3) & 1) * 32 + (p & 31)) * 8 + (e & 7);
}
__device__ __forceinline__ size_t val_at(const Dims& d, int p, int e) {
  const int a = (p & 31) >> 3, g = (p >> 2) & 1;     // key 8 a + 4 g + b of the tile: step a / 2, element 4 (a % 2) + b
  return (((size_t)(p >> 5) * d.NC * d.LT + (e >> 5)) * 2 + (a >> 1)) * 512 + (g * 32 + (e & 31)) * 8 + (a & 1) * 4 + (p & 3);
}

// ---- new cache rows ------------------------------------------------------------------------------
// One block of 256 threads per token.
template <int NC>
__device__ __forceinline__ void fill_row(const float* __restrict__ u, const tlhip_latent_attn& a, int p, float* red) {
  const Dims d = dims_of(a);
  const int tid = threadIdx.x;
  const float* x = u + a.kv_off;
  float ss = 0.f;
  for (int i = tid; i < d.L; i += 256) ss = fmaf(x[i], x[i], ss);
  const float inv = 1.0f / sqrtf(block_sum<4>(ss, red) / (float)d.L + a.eps);
  uint16_t* kc = static_cast<uint16_t*>(a.keys);
  uint16_t* vc = static_cast<uint16_t*>(a.values);
  const float2* tab = static_cast<const float2*>(a.angles) + (size_t)p * (d.R / 2);
  for (int i = tid; i < d.L + d.R; i += 256) {
    float v;
    if (i < d.L) v = x[i] * inv * static_cast<const float*>(a.kv_norm)[i];
    else {
      const int r = i - d.L, half = d.R / 2, j = r < half ? r : r - half;
      const float2 cs = tab[j];
      const float lo = x[d.L + j], hi = x[d.L + half + j];
      v = r < half ? lo * cs.x - hi * cs.y : hi * cs.x + lo * cs.y;
    }
    uint16_t t[NC];
    cut<NC>(v, t);
    const size_t k = key_at(d, p, i);
#pragma unroll
    for (int n = 0; n < NC; n++) kc[k + (size_t)n * d.DS * 512] = t[n];
    if (i < d.L) {
      const size_t w = val_at(d, p, i);
#pragma unroll
      for (int n = 0; n < NC; n++) vc[w + (size_t)n * d.LT * 1024] = t[n];
    }
  }
}

// ---- queries -------------------------------------------------------------------------------------
// Image of a tile of 32 query rows (row = token * heads + head): [term][DS][lane][8], scaled by
// scale * log2 e before it is cut. Block (slice of 128 dims, head, TQ tokens), 256 threads: 16 dim units of 8 x
// 16 groups of query dims. Blocks past the slices fill the cache rows (one per token).
constexpr int kSliceDims = 128;
template <int TQ, int NC, int NQ>
__global__ __launch_bounds__(256) void latent_query_kernel(const float* __restrict__ u, int64_t ldu, const float* __restrict__ q,
                                                           int64_t ldq, const tlhip_latent_attn a, uint16_t* __restrict__ qimg,
                                                           int T, int pos0, const uint32_t* __restrict__ d_pos, int slices) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const Dims d = dims_of(a);
  const int tid = threadIdx.x, p0 = d_pos ? (int)*d_pos : pos0;
  const int tiles = (T + TQ - 1) / TQ, work = slices * d.H * tiles;
  if ((int)blockIdx.x >= work) {
    const int t = (int)blockIdx.x - work;
    fill_row<NC>(u + (size_t)t * ldu, a, p0 + t, lds);
    return;
  }
  const int slice = blockIdx.x % slices, h = blockIdx.x / slices % d.H, t0 = blockIdx.x / slices / d.H * TQ;
  const int nt = min(TQ, T - t0), unit = slice * (kSliceDims / 8) + (tid & 15), dg = tid >> 4, ldk = up8(d.L);
  float* qs = lds;                     // [TQ][D] unrotated query dims
  float* red = lds + TQ * d.D;         // [16 groups][16 units][8] per token
  for (int i = tid; i < TQ * d.D; i += 256) {
    const int t = i / d.D;
    qs[i] = q[(size_t)(t0 + min(t, nt - 1)) * ldq + h * (d.D + d.R) + i % d.D];
  }
  __syncthreads();
  float acc[TQ][8];
#pragma unroll
  for (int t = 0; t < TQ; t++)
#pragma unroll
    for (int j = 0; j < 8; j++) acc[t][j] = 0.f;
  if (unit * 8 < ldk) {
    const u32x4* w = reinterpret_cast<const u32x4*>(static_cast<const uint16_t*>(a.uk) + (size_t)h * d.D * ldk) + unit;
    const int n8 = ldk / 8;
#pragma unroll 4
    for (int k = dg; k < d.D; k += 16) {
      const u32x4 x = w[(size_t)k * n8];
#pragma unroll
      for (int t = 0; t < TQ; t++) {
        const float f = qs[t * d.D + k];
#pragma unroll
        for (int j = 0; j < 4; j++) {
          acc[t][2 * j] = fmaf(bf16_lo(x[j]), f, acc[t][2 * j]);
          acc[t][2 * j + 1] = fmaf(bf16_hi(x[j]), f, acc[t][2 * j + 1]);
        }
      }
    }
  }
  const float sc = a.scale * 1.4426950408889634f;
  for (int t = 0; t < TQ; t++) {
    if (t >= nt) break;
#pragma unroll
    for (int tt = 0; tt < TQ; tt++)
      if (tt == t) {
#pragma unroll
        for (int j = 0; j < 8; j++) red[(dg * 16 + (tid & 15)) * 8 + j] = acc[tt][j];
      }
    __syncthreads();
    if (tid < 128) {                   // dim `e` of the slice
      const int e = slice * kSliceDims + tid;
      float v = 0.f;
      if (e < d.L) {
#pragma unroll
        for (int k = 0; k < 16; k++) v += red[k * 128 + tid];
      } else if (e < d.L + d.R) {
        const int r = e - d.L, half = d.R / 2, j = r < half ? r : r - half;
        const float2 cs = static_cast<const float2*>(a.angles)[(size_t)(p0 + t0 + t) * half + j];
        const float* x = q + (size_t)(t0 + t) * ldq + h * (d.D + d.R) + d.D;
        v = r < half ? x[j] * cs.x - x[half + j] * cs.y : x[half + j] * cs.x + x[j] * cs.y;
      }
      if (e < d.DS * 16) {
        uint16_t o[NQ];
        cut<NQ>(v * sc, o);
        const int row = (t0 + t) * d.H + h;
        const size_t at = ((size_t)(row >> 5) * NQ * d.DS + (e >> 4)) * 512 + (((e >> 3) & 1) * 32 + (row & 31)) * 8 + (e & 7);
#pragma unroll
        for (int n = 0; n < NQ; n++) qimg[at + (size_t)n * d.DS * 512] = o[n];
      }
    }
    __syncthreads();
  }
}

// The same for chunks on the matrix cores: C^T = uk_h^T qn^T, queries in two bf16 terms. Blocks: (slice of 128 latent dims,
// head, 128 tokens), a wavefront per 32 tokens; then rotated parts and padding (256 numbers a block); then cache rows.
// LDS: the slice of uk_h as operand fragments [4 tiles of 32 dims][KST steps of 16][lane][8].
constexpr int kQTok = 128;
template <bool VEC>
__device__ __forceinline__ void query_frag(const float* __restrict__ x, int k, int D, u32x4 (&f)[2]) {
  float v[8];
  if (VEC && k + 8 <= D) {
    const f32x4 lo = *reinterpret_cast<const f32x4*>(x + k), hi = *reinterpret_cast<const f32x4*>(x + k + 4);
#pragma unroll
    for (int j = 0; j < 4; j++) { v[j] = lo[j]; v[4 + j] = hi[j]; }
  } else {
#pragma unroll
    for (int j = 0; j < 8; j++) {
      const float t = x[min(k + j, D - 1)];
      v[j] = k + j < D ? t : 0.f;
    }
  }
#pragma unroll
  for (int j = 0; j < 4; j++) {
    uint16_t a[2], b[2];
    cut<2>(v[2 * j], a);
    cut<2>(v[2 * j + 1], b);
#pragma unroll
    for (int n = 0; n < 2; n++) f[n][j] = (uint32_t)a[n] | ((uint32_t)b[n] << 16);
  }
}
template <bool VEC>
__global__ __launch_bounds__(256) void latent_query_mfma_kernel(const float* __restrict__ u, int64_t ldu, const float* __restrict__ q,
                                                                int64_t ldq, const tlhip_latent_attn a, uint16_t* __restrict__ qimg,
                                                                int T, int pos0, int slices, int tail_blocks) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const Dims d = dims_of(a);
  const int tid = threadIdx.x, groups = (T + kQTok - 1) / kQTok, work = slices * d.H * groups;
  const float sc = a.scale * 1.4426950408889634f;
  const auto image_at = [&](int row, int e) {
    return ((size_t)(row >> 5) * 2 * d.DS + (e >> 4)) * 512 + (((e >> 3) & 1) * 32 + (row & 31)) * 8 + (e & 7);
  };
  if ((int)blockIdx.x >= work + tail_blocks) {
    const int t = (int)blockIdx.x - work - tail_blocks;
    fill_row<1>(u + (size_t)t * ldu, a, pos0 + t, lds);
    return;
  }
  if ((int)blockIdx.x >= work) {       // a pair of rotated dims, or a number of the padding
    const int half = d.R / 2, pad = d.DS * 16 - d.L - d.R, items = half + pad;
    const int64_t i = (int64_t)((int)blockIdx.x - work) * 256 + tid;
    if (i >= (int64_t)T * d.H * items) return;
    const int j = (int)(i % items), row = (int)(i / items), t = row / d.H, h = row - t * d.H;
    const auto put = [&](int e, float v) {
      uint16_t o[2];
      cut<2>(v, o);
      const size_t at = image_at(row, e);
      qimg[at] = o[0];
      qimg[at + (size_t)d.DS * 512] = o[1];
    };
    if (j >= half) {
      put(d.L + d.R + j - half, 0.f);
      return;
    }
    const float2 cs = static_cast<const float2*>(a.angles)[(size_t)(pos0 + t) * half + j];
    const float* x = q + (size_t)t * ldq + h * (d.D + d.R) + d.D;
    const float lo = x[j], hi = x[half + j];
    put(d.L + j, (lo * cs.x - hi * cs.y) * sc);
    put(d.L + half + j, (hi * cs.x + lo * cs.y) * sc);
    return;
  }
  // a line of the image holds rows of adjacent heads: their blocks on one die, where its L2 joins the stores
  const int id = work % 8 == 0 ? (int)(blockIdx.x % 8) * (work / 8) + (int)blockIdx.x / 8 : (int)blockIdx.x;
  const int h = id % d.H, slice = id / d.H % slices, t0 = id / d.H / slices * kQTok;
  const int KST = (d.D + 15) / 16, ldk = up8(d.L);
  u32x4* frag = reinterpret_cast<u32x4*>(lds);
  for (int i = tid; i < 16 * 2 * KST; i += 256) {        // 8 latent dims x 8 query dims, transposed
    const int e8 = i & 15, k8 = i >> 4, e = slice * kSliceDims + 8 * e8;
    u32x4 x[8];
#pragma unroll
    for (int k = 0; k < 8; k++) {
      x[k] = u32x4{0, 0, 0, 0};
      if (8 * k8 + k < d.D && e < ldk)
        x[k] = *reinterpret_cast<const u32x4*>(static_cast<const uint16_t*>(a.uk) + ((size_t)h * d.D + 8 * k8 + k) * ldk + e);
    }
#pragma unroll
    for (int n = 0; n < 8; n++) {
      u32x4 o;
#pragma unroll
      for (int j = 0; j < 4; j++) {
        const uint32_t lo = x[2 * j][n >> 1], hi = x[2 * j + 1][n >> 1];
        o[j] = n & 1 ? (lo >> 16) | (hi & 0xffff0000u) : (lo & 0xffffu) | (hi << 16);
      }
      const int c = 8 * e8 + n;
      frag[((c >> 5) * KST + (k8 >> 1)) * 64 + (k8 & 1) * 32 + (c & 31)] = o;
    }
  }
  __syncthreads();
  const int lane = tid & 63, g = lane >> 5, c = lane & 31, t = t0 + (tid >> 6) * 32 + c;
  const float* x = q + (size_t)min(t, T - 1) * ldq + h * (d.D + d.R);
  f32x16 acc[4];
#pragma unroll
  for (int m = 0; m < 4; m++)
#pragma unroll
    for (int v = 0; v < 16; v++) acc[m][v] = 0.f;
  u32x4 nf[2];
  query_frag<VEC>(x, 8 * g, d.D, nf);
  for (int st = 0; st < KST; st++) {
    const u32x4 qf[2] = {nf[0], nf[1]};
    query_frag<VEC>(x, min(16 * st + 16, 16 * KST - 16) + 8 * g, d.D, nf);
#pragma unroll
    for (int m = 0; m < 4; m++) {
      const bf16x8 k = __builtin_bit_cast(bf16x8, frag[(m * KST + st) * 64 + lane]);
      acc[m] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(k, __builtin_bit_cast(bf16x8, qf[1]), acc[m], 0, 0, 0);
      acc[m] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(k, __builtin_bit_cast(bf16x8, qf[0]), acc[m], 0, 0, 0);
    }
  }
  if (t >= T) return;
  const int row = t * d.H + h;
#pragma unroll
  for (int m = 0; m < 4; m++)
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const int e = slice * kSliceDims + 32 * m + 8 * i + 4 * g;
      uint16_t o[4][2];
#pragma unroll
      for (int b = 0; b < 4; b++) cut<2>(acc[m][4 * i + b] * sc, o[b]);
#pragma unroll
      for (int n = 0; n < 2; n++) {
        uint16_t* at = qimg + image_at(row, e) + (size_t)n * d.DS * 512;
        if (e + 4 <= d.L)
          *reinterpret_cast<u32x2*>(at) = u32x2{(uint32_t)o[0][n] | ((uint32_t)o[1][n] << 16), (uint32_t)o[2][n] | ((uint32_t)o[3][n] << 16)};
        else
#pragma unroll
          for (int b = 0; b < 4; b++)
            if (e + b < d.L) at[b] = o[b][n];
      }
    }
}

// ---- attention -----------------------------------------------------------------------------------
// Partials per (split, row): m [S][rows], l [S][rows], acc [S][rows][32 LT].
// Block (query tile, split) of eight wavefronts, 64 keys at a time: pairs of key tiles split, split + S, ...
// Scores: wavefront (k, d) takes key tile k and every fourth dim step from d, its queries in registers; the four
// partial tiles meet in LDS and d's owner keeps eight keys of a lane pair: maximum, weights (two bf16 terms, half an
// operand fragment) and sum are formed once. Values: wavefront w takes value tiles w, w + 8, ... (NL of them).
template <int KS, int NL>
__global__ __launch_bounds__(512) void latent_attend_kernel(const tlhip_latent_attn a, const uint16_t* __restrict__ qimg,
                                                            float* __restrict__ part, int T, int pos0,
                                                            const uint32_t* __restrict__ d_pos, int S, int rows) {
  __shared__ f32x4 ex[8][4][64];       // partial scores of (wavefront, eight keys)
  __shared__ u32x4 pb[4][2][64];       // weights of (16 keys, term)
  __shared__ float mx[8][32];
  const Dims d = dims_of(a);
  const int tid = threadIdx.x, lane = tid & 63, g = lane >> 5, c = lane & 31;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6), kt = wave & 1, dq = wave >> 1;
  const int rt = blockIdx.x / S, split = blockIdx.x % S;
  const int p0 = d_pos ? (int)*d_pos : pos0;
  const int row = rt * 32 + c;                       // this lane's query row
  const int limit = row < T * d.H ? p0 + row / d.H : -1;
  const int last = p0 + min(rt * 32 + 31, T * d.H - 1) / d.H, ntiles = last / 32 + 1, npairs = (ntiles + 1) / 2;
  const u32x4* kc = reinterpret_cast<const u32x4*>(a.keys) + lane;
  const u32x4* vc = reinterpret_cast<const u32x4*>(a.values) + lane;
  const u32x4* qg = reinterpret_cast<const u32x4*>(qimg) + (size_t)rt * 2 * d.DS * 64 + lane;

  u32x4 kr[KS], qr[KS][2];
  const auto load_keys = [&](int pair) {             // (steps past the last: any key meets a zero query)
    const u32x4* k = kc + (size_t)min(2 * pair + kt, ntiles - 1) * d.DS * 64;
#pragma unroll
    for (int i = 0; i < KS; i++) kr[i] = k[min(dq + 4 * i, d.DS - 1) * 64];
  };
  load_keys(split);
#pragma unroll
  for (int i = 0; i < KS; i++)
#pragma unroll
    for (int n = 0; n < 2; n++) {
      const u32x4 x = qg[(n * d.DS + min(dq + 4 * i, d.DS - 1)) * 64];
      qr[i][n] = dq + 4 * i < d.DS ? x : u32x4{0, 0, 0, 0};
    }
  f32x16 o[NL];
#pragma unroll
  for (int i = 0; i < NL; i++)
#pragma unroll
    for (int v = 0; v < 16; v++) o[i][v] = 0.f;
  float m = -INFINITY, l = 0.f;
  for (int pair = split; pair < npairs; pair += S) {
    u32x4 vr[NL][4];                   // values of these keys, requested before the scores are formed
#pragma unroll
    for (int i = 0; i < NL; i++)
#pragma unroll
      for (int k = 0; k < 4; k++)
        vr[i][k] = vc[(((size_t)min(2 * pair + (k >> 1), ntiles - 1) * d.LT + min(wave + 8 * i, d.LT - 1)) * 2 + (k & 1)) * 64];
    f32x16 s[2];
#pragma unroll
    for (int n = 0; n < 2; n++)
#pragma unroll
      for (int v = 0; v < 16; v++) s[n][v] = 0.f;
#pragma unroll
    for (int i = 0; i < KS; i++)
#pragma unroll
      for (int n = 1; n >= 0; n--)
        s[n] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, kr[i]), __builtin_bit_cast(bf16x8, qr[i][n]), s[n], 0, 0, 0);
    load_keys(min(pair + S, npairs - 1));
#pragma unroll
    for (int i = 0; i < 4; i++)
      ex[wave][i][lane] = f32x4{s[0][4 * i] + s[1][4 * i], s[0][4 * i + 1] + s[1][4 * i + 1], s[0][4 * i + 2] + s[1][4 * i + 2],
                                s[0][4 * i + 3] + s[1][4 * i + 3]};
    __syncthreads();
    f32x4 e = ex[kt][dq][lane];
#pragma unroll
    for (int w = 1; w < 4; w++) e += ex[2 * w + kt][dq][lane];
#pragma unroll
    for (int b = 0; b < 4; b++)
      if (64 * pair + 32 * kt + 8 * dq + 4 * g + b > limit) e[b] = -INFINITY;
    const float mt = fmaxf(fmaxf(e[0], e[1]), fmaxf(e[2], e[3]));
    const LanePair pr = swap32(mt, mt);
    if (g == 0) mx[wave][c] = fmaxf(pr.first, pr.second);
    __syncthreads();
    float mn = m;
#pragma unroll
    for (int w = 0; w < 8; w++) mn = fmaxf(mn, mx[w][c]);
    const float mz = mn == -INFINITY ? 0.f : mn;
    const float f = exp2f(m - mz);                   // (m = -inf: 0)
    m = mn;
    uint16_t p[4][2];
    float sum = 0.f;
#pragma unroll
    for (int b = 0; b < 4; b++) {
      const float w = exp2f(e[b] - mz);
      sum += w;
      cut<2>(w, p[b]);
    }
    l = fmaf(l, f, sum);                             // this lane's keys
#pragma unroll
    for (int n = 0; n < 2; n++)
      reinterpret_cast<u32x2*>(&pb[2 * kt + (dq >> 1)][n][lane])[dq & 1] =
          u32x2{(uint32_t)p[0][n] | ((uint32_t)p[1][n] << 16), (uint32_t)p[2][n] | ((uint32_t)p[3][n] << 16)};
    if (__any(f != 1.f))
#pragma unroll
      for (int i = 0; i < NL; i++)
#pragma unroll
        for (int v = 0; v < 16; v++) o[i][v] *= f;
    __syncthreads();
#pragma unroll
    for (int k = 0; k < 4; k++)
#pragma unroll
      for (int n = 1; n >= 0; n--) {
        const bf16x8 pf = __builtin_bit_cast(bf16x8, pb[k][n][lane]);
#pragma unroll
        for (int i = 0; i < NL; i++)
          o[i] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, vr[i][k]), pf, o[i], 0, 0, 0);
      }
  }
  const LanePair lp = swap32(l, l);
  __syncthreads();                     // mx has been read
  if (g == 0) mx[wave][c] = lp.first + lp.second;
  __syncthreads();
  const size_t R = (size_t)rows, at = (size_t)split * R + row;
  float* pm = part;
  float* pl = part + (size_t)S * R;
  float* pa = pl + (size_t)S * R;
  if (wave == 0 && g == 0) {
    float t = mx[0][c];
#pragma unroll
    for (int w = 1; w < 8; w++) t += mx[w][c];
    pm[at] = m;
    pl[at] = t;
  }
#pragma unroll
  for (int i = 0; i < NL; i++) {
    const int lt = wave + 8 * i;
    if (lt < d.LT)
#pragma unroll
      for (int k = 0; k < 4; k++)
        *reinterpret_cast<f32x4*>(pa + at * (32 * d.LT) + 32 * lt + 8 * k + 4 * g) = f32x4{o[i][4 * k], o[i][4 * k + 1], o[i][4 * k + 2], o[i][4 * k + 3]};
  }
}

// Every term against every term. Four wavefronts; key tiles split, split + S, ... Scores: every wavefront takes each
// fourth dim step, the four partial sums meet in LDS and every wavefront adds them in the same order. Values:
// wavefront w takes value tiles w, w + 4, ... (NL of them).
template <int NL, int NC, int NQ>
__global__ __launch_bounds__(256) void latent_attend_exact_kernel(const tlhip_latent_attn a, const uint16_t* __restrict__ qimg,
                                                            float* __restrict__ part, int T, int pos0,
                                                            const uint32_t* __restrict__ d_pos, int S, int rows) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const Dims d = dims_of(a);
  const int tid = threadIdx.x, lane = tid & 63, g = lane >> 5, c = lane & 31;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int rt = blockIdx.x / S, split = blockIdx.x % S;
  const int p0 = d_pos ? (int)*d_pos : pos0;
  const int row = rt * 32 + c;                       // this lane's query row
  const int limit = row < T * d.H ? p0 + row / d.H : -1;
  const int last = p0 + min(rt * 32 + 31, T * d.H - 1) / d.H, ntiles = last / 32 + 1;   // key tiles the tile's last row sees
  u32x4* qs = reinterpret_cast<u32x4*>(lds);         // [NQ][DS][64]
  f32x4* red = reinterpret_cast<f32x4*>(qs + NQ * d.DS * 64);   // [2][4 waves][4][64]
  const u32x4* qg = reinterpret_cast<const u32x4*>(qimg) + (size_t)rt * NQ * d.DS * 64;
  for (int i = tid; i < NQ * d.DS * 64; i += 256) qs[i] = qg[i];
  const u32x4* kc = reinterpret_cast<const u32x4*>(a.keys) + lane;
  const u32x4* vc = reinterpret_cast<const u32x4*>(a.values) + lane;

  f32x16 o[NL];
#pragma unroll
  for (int i = 0; i < NL; i++)
#pragma unroll
    for (int v = 0; v < 16; v++) o[i][v] = 0.f;
  float m = -INFINITY, l = 0.f;
  __syncthreads();
  int par = 0;
  for (int tile = split; tile < ntiles; tile += S, par ^= 1) {
    // values of this tile, requested before the scores are formed
    u32x4 vr[NL][NC][2];
#pragma unroll
    for (int i = 0; i < NL; i++)
#pragma unroll
      for (int n = 0; n < NC; n++)
#pragma unroll
        for (int k = 0; k < 2; k++) {
          const int lt = min(wave + 4 * i, d.LT - 1);
          vr[i][n][k] = vc[((((size_t)tile * NC + n) * d.LT + lt) * 2 + k) * 64];
        }
    f32x16 s;
#pragma unroll
    for (int v = 0; v < 16; v++) s[v] = 0.f;
    for (int st = wave; st < d.DS; st += 4) {
      u32x4 kr[NC], qr[NQ];
#pragma unroll
      for (int n = 0; n < NC; n++) kr[n] = kc[(((size_t)tile * NC + n) * d.DS + st) * 64];
#pragma unroll
      for (int n = 0; n < NQ; n++) qr[n] = qs[(n * d.DS + st) * 64 + lane];
#pragma unroll
      for (int n = NC - 1; n >= 0; n--)
#pragma unroll
        for (int k = NQ - 1; k >= 0; k--)
          s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, kr[n]), __builtin_bit_cast(bf16x8, qr[k]), s, 0, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < 4; i++)
      red[((par * 4 + wave) * 4 + i) * 64 + lane] = f32x4{s[4 * i], s[4 * i + 1], s[4 * i + 2], s[4 * i + 3]};
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 4; i++) {
      f32x4 t = red[(par * 16 + i) * 64 + lane];
#pragma unroll
      for (int w = 1; w < 4; w++) t += red[(par * 16 + 4 * w + i) * 64 + lane];
#pragma unroll
      for (int b = 0; b < 4; b++) s[4 * i + b] = tile * 32 + 8 * i + 4 * g + b <= limit ? t[b] : -INFINITY;
    }
    float mt = s[0];
#pragma unroll
    for (int v = 1; v < 16; v++) mt = fmaxf(mt, s[v]);
    const LanePair pr = swap32(mt, mt);
    const float mn = fmaxf(m, fmaxf(pr.first, pr.second)), mz = mn == -INFINITY ? 0.f : mn;
    const float f = exp2f(m - mz);                   // (m = -inf: 0)
    float sum = 0.f;
    uint16_t p[16][NQ];
#pragma unroll
    for (int v = 0; v < 16; v++) {
      const float e = exp2f(s[v] - mz);
      sum += e;
      cut<NQ>(e, p[v]);
    }
    l = fmaf(l, f, sum);                             // this lane's half of the keys
    m = mn;
#pragma unroll
    for (int i = 0; i < NL; i++)
#pragma unroll
      for (int v = 0; v < 16; v++) o[i][v] *= f;
#pragma unroll
    for (int k = 0; k < 2; k++) {
      u32x4 pf[NQ];
#pragma unroll
      for (int n = 0; n < NQ; n++)
#pragma unroll
        for (int j = 0; j < 4; j++) pf[n][j] = (uint32_t)p[8 * k + 2 * j][n] | ((uint32_t)p[8 * k + 2 * j + 1][n] << 16);
#pragma unroll
      for (int i = 0; i < NL; i++)
#pragma unroll
        for (int n = NC - 1; n >= 0; n--)
#pragma unroll
          for (int q = NQ - 1; q >= 0; q--)
            o[i] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, vr[i][n][k]), __builtin_bit_cast(bf16x8, pf[q]), o[i], 0, 0, 0);
    }
  }
  const LanePair lp = swap32(l, l);
  l = lp.first + lp.second;
  const size_t R = (size_t)rows, at = (size_t)split * R + row;
  float* pm = part;
  float* pl = part + (size_t)S * R;
  float* pa = pl + (size_t)S * R;
  if (wave == 0 && g == 0) {
    pm[at] = m;
    pl[at] = l;
  }
#pragma unroll
  for (int i = 0; i < NL; i++) {
    const int lt = wave + 4 * i;
    if (lt < d.LT)
#pragma unroll
      for (int q = 0; q < 4; q++)
        *reinterpret_cast<f32x4*>(pa + at * (32 * d.LT) + 32 * lt + 8 * q + 4 * g) = f32x4{o[i][4 * q], o[i][4 * q + 1], o[i][4 * q + 2], o[i][4 * q + 3]};
  }
}

// ---- splits joined, values' up-projection, gate ---------------------------------------------------
// Block (slice of kOutRows value rows, head, TQ <= 4 tokens) of NT threads; G groups of threads share the splits.
constexpr int kMaxSplits = 64;
constexpr int kOutRows = 32;
__host__ __device__ inline int out_groups(int NT, int TQ, int LV) { const int n = TQ * (LV / 4); return n >= NT ? 1 : NT / n; }
template <int TQ, int NT>
__global__ __launch_bounds__(NT) void latent_out_kernel(const float* __restrict__ u, int64_t ldu, float* __restrict__ y, int64_t ldy,
                                                        const tlhip_latent_attn a, const float* __restrict__ part, int T, int S,
                                                        int rows, int slices) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  constexpr int NW = NT / 64;
  const Dims d = dims_of(a);
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int slice = blockIdx.x % slices, h = blockIdx.x / slices % d.H, t0 = blockIdx.x / slices / d.H * TQ;
  const int nt = min(TQ, T - t0), LV = 32 * d.LT, ldv = up8(d.L), n8 = ldv / 8, G = out_groups(NT, TQ, LV), items = TQ * (LV / 4);
  float* oc = lds;                     // [G][TQ][LV] sums of latents, normalised
  float* w = oc + G * TQ * LV;         // [TQ][S] the splits' weights
  const size_t R = (size_t)rows;
  const float *pm = part, *pl = part + (size_t)S * R, *pa = pl + (size_t)S * R;
  const int v1 = min(d.V, (slice + 1) * kOutRows), vw = slice * kOutRows + wave;
  const u32x4* uv = reinterpret_cast<const u32x4*>(static_cast<const uint16_t*>(a.uv)) + (size_t)h * d.V * n8;
  constexpr int PRE = kOutRows / NW < 2 ? 1 : 2;     // rows whose weights are requested up front
  u32x4 pre[PRE];
  float gate[PRE];                     // (of a single token)
#pragma unroll
  for (int i = 0; i < PRE; i++) {
    const int v = min(vw + i * NW, d.V - 1);
    pre[i] = uv[(size_t)v * n8 + min(lane, n8 - 1)];
    gate[i] = TQ == 1 && a.gate_off >= 0 ? u[(size_t)t0 * ldu + a.gate_off + h * d.V + v] : 0.f;
  }
  f32x4 v[8];                          // eight splits' latents of this thread's item, the first ones before the weights are known
  const auto load_splits = [&](int i, int s0) {
    const int j = i % items, t = j / (LV / 4), e = 4 * (j - t * (LV / 4));
    const float* src = pa + ((size_t)(t0 + min(t, nt - 1)) * d.H + h) * LV + e;
#pragma unroll
    for (int k = 0; k < 8; k++) v[k] = *reinterpret_cast<const f32x4*>(src + (size_t)min(s0 + k * G, S - 1) * R * LV);
  };
  load_splits(tid, tid / items);
  if (wave < TQ) {                     // a wavefront weighs the (up to 64) splits of one token
    const int row = (t0 + min(wave, nt - 1)) * d.H + h;
    const float m = lane < S ? pm[lane * R + row] : -INFINITY, l = lane < S ? pl[lane * R + row] : 0.f;
    const float f = exp2f(m - wave_max(m)), tot = wave_sum(f * l);
    if (lane < S) w[wave * S + lane] = f / tot;
  }
  __syncthreads();
  for (int i = tid; i < items * G; i += NT) {
    const int grp = i / items, j = i - grp * items, t = j / (LV / 4), e = 4 * (j - t * (LV / 4));
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    for (int s0 = grp; s0 < S; s0 += 8 * G) {
      if (i != tid || s0 != grp) load_splits(i, s0);
#pragma unroll
      for (int k = 0; k < 8; k++)
        if (s0 + k * G < S) {
          const float f = w[t * S + s0 + k * G];
          acc += v[k] * f;
        }
    }
    *reinterpret_cast<f32x4*>(oc + grp * TQ * LV + t * LV + e) = acc;
  }
  __syncthreads();
  if (G > 1) {
    for (int i = tid; i < TQ * LV; i += NT) {
      float t = oc[i];
      for (int k = 1; k < G; k++) t += oc[k * TQ * LV + i];
      oc[i] = t;
    }
    __syncthreads();
  }
  for (int v = vw, i = 0; v < v1; v += NW, i++) {
    float acc[TQ];
#pragma unroll
    for (int t = 0; t < TQ; t++) acc[t] = 0.f;
    for (int k = lane; k < n8; k += 64) {
      u32x4 x;
      if (k == lane && i < PRE) {
        x = pre[0];
        if (PRE > 1 && i == 1) x = pre[PRE - 1];
      } else {
        x = uv[(size_t)v * n8 + k];
      }
#pragma unroll
      for (int t = 0; t < TQ; t++) {
        const f32x4 c0 = *reinterpret_cast<const f32x4*>(oc + t * LV + 8 * k), c1 = *reinterpret_cast<const f32x4*>(oc + t * LV + 8 * k + 4);
        acc[t] = fmaf(bf16_lo(x[0]), c0[0], acc[t]);
        acc[t] = fmaf(bf16_hi(x[0]), c0[1], acc[t]);
        acc[t] = fmaf(bf16_lo(x[1]), c0[2], acc[t]);
        acc[t] = fmaf(bf16_hi(x[1]), c0[3], acc[t]);
        acc[t] = fmaf(bf16_lo(x[2]), c1[0], acc[t]);
        acc[t] = fmaf(bf16_hi(x[2]), c1[1], acc[t]);
        acc[t] = fmaf(bf16_lo(x[3]), c1[2], acc[t]);
        acc[t] = fmaf(bf16_hi(x[3]), c1[3], acc[t]);
      }
    }
#pragma unroll
    for (int t = 0; t < TQ; t++) {
      const float s = wave_sum(acc[t]);
      if (lane == 0 && t < nt) {
        float o = s;
        if (a.gate_off >= 0) {
          float z;
          if (TQ == 1 && i < PRE) z = i == 0 ? gate[0] : gate[PRE - 1];
          else z = u[(size_t)(t0 + t) * ldu + a.gate_off + h * d.V + v];
          o = s / (1.f + expf(-z));
        }
        y[(size_t)(t0 + t) * ldy + a.y_off + h * d.V + v] = o;
      }
    }
  }
}

// The same for chunks on the matrix cores: block (head, 32 tokens) of 256 threads, y^T = uv_h oc^T with the joined
// latents in two bf16 terms as operand fragments in LDS [KST steps of 16][term][lane][8]; a wavefront per 32 values.
// VEC: rows of u and y take 16-byte accesses.
template <bool VEC>
__global__ __launch_bounds__(256) void latent_out_mfma_kernel(const float* __restrict__ u, int64_t ldu, float* __restrict__ y, int64_t ldy,
                                                              const tlhip_latent_attn a, const float* __restrict__ part, int T, int S,
                                                              int rows) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const Dims d = dims_of(a);
  const int tid = threadIdx.x, lane = tid & 63, g = lane >> 5, c = lane & 31;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = blockIdx.x % d.H, t0 = blockIdx.x / d.H * 32, nt = min(32, T - t0);
  const int LV = 32 * d.LT, KST = 2 * d.LT, ldv = up8(d.L);
  u32x4* frag = reinterpret_cast<u32x4*>(lds);
  float* w = lds + (size_t)KST * 512;  // [32][S] the splits' weights
  const size_t R = (size_t)rows;
  const float *pm = part, *pl = part + (size_t)S * R, *pa = pl + (size_t)S * R;
  if (S == 1) {
    if (tid < 32) w[tid] = 1.f / pl[(t0 + min(tid, nt - 1)) * d.H + h];
  } else {
    for (int t = wave; t < 32; t += 4) {
      const int row = (t0 + min(t, nt - 1)) * d.H + h;
      const float m = lane < S ? pm[lane * R + row] : -INFINITY, l = lane < S ? pl[lane * R + row] : 0.f;
      const float f = exp2f(m - wave_max(m)), tot = wave_sum(f * l);
      if (lane < S) w[t * S + lane] = f / tot;
    }
  }
  __syncthreads();
  for (int i = tid; i < 32 * 2 * KST; i += 256) {        // 8 latent dims of a token; 16 tokens x 4 runs to a wavefront
    const int t = ((i >> 2) & 15) + 16 * ((i >> 6) & 1), r = (i & 3) + 4 * (i >> 7);
    const float* src = pa + ((size_t)(t0 + min(t, nt - 1)) * d.H + h) * LV + 8 * r;
    f32x4 lo = {0.f, 0.f, 0.f, 0.f}, hi = lo;
    for (int s = 0; s < S; s++) {
      const float f = w[t * S + s];
      lo += *reinterpret_cast<const f32x4*>(src + (size_t)s * R * LV) * f;
      hi += *reinterpret_cast<const f32x4*>(src + (size_t)s * R * LV + 4) * f;
    }
    u32x4 o[2];
#pragma unroll
    for (int j = 0; j < 4; j++) {
      uint16_t x[2], z[2];
      cut<2>(j < 2 ? lo[2 * j] : hi[2 * j - 4], x);
      cut<2>(j < 2 ? lo[2 * j + 1] : hi[2 * j - 3], z);
#pragma unroll
      for (int n = 0; n < 2; n++) o[n][j] = (uint32_t)x[n] | ((uint32_t)z[n] << 16);
    }
#pragma unroll
    for (int n = 0; n < 2; n++) frag[((r >> 1) * 2 + n) * 64 + (r & 1) * 32 + t] = o[n];
  }
  __syncthreads();
  const uint16_t* uv = static_cast<const uint16_t*>(a.uv) + (size_t)h * d.V * ldv;
  for (int vt = wave; 32 * vt < d.V; vt += 4) {
    const uint16_t* wr = uv + (size_t)min(32 * vt + c, d.V - 1) * ldv;
    f32x16 acc;
#pragma unroll
    for (int v = 0; v < 16; v++) acc[v] = 0.f;
    const auto weights = [&](int st) -> u32x4 {
      const int k = 16 * st + 8 * g;
      const u32x4 x = *reinterpret_cast<const u32x4*>(wr + min(k, ldv - 8));
      return k < ldv ? x : u32x4{0, 0, 0, 0};
    };
    u32x4 x[2] = {weights(0), weights(1)};
    for (int s0 = 0; s0 < KST; s0 += 2) {
      u32x4 nx[2] = {weights(min(s0 + 2, KST - 2)), weights(min(s0 + 3, KST - 1))};
#pragma unroll
      for (int k = 0; k < 2; k++) {
#pragma unroll
        for (int n = 1; n >= 0; n--)
          acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, x[k]),
                                                        __builtin_bit_cast(bf16x8, frag[((s0 + k) * 2 + n) * 64 + lane]), acc, 0, 0, 0);
        x[k] = nx[k];
      }
    }
    if (c >= nt) continue;
    const float* gate = u + (size_t)(t0 + c) * ldu + a.gate_off + h * d.V;
    float* out = y + (size_t)(t0 + c) * ldy + a.y_off + h * d.V;
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const int v = 32 * vt + 8 * i + 4 * g;
      f32x4 o = {acc[4 * i], acc[4 * i + 1], acc[4 * i + 2], acc[4 * i + 3]};
      if (VEC && v + 4 <= d.V) {
        if (a.gate_off >= 0) {
          const f32x4 z = *reinterpret_cast<const f32x4*>(gate + v);
#pragma unroll
          for (int b = 0; b < 4; b++) o[b] = o[b] / (1.f + expf(-z[b]));
        }
        *reinterpret_cast<f32x4*>(out + v) = o;
      } else {
#pragma unroll
        for (int b = 0; b < 4; b++)
          if (v + b < d.V) out[v + b] = a.gate_off >= 0 ? o[b] / (1.f + expf(-gate[v + b])) : o[b];
      }
    }
  }
}

static int check(const tlhip_latent_attn* a, const char* who) {
  if (!a || a->heads <= 0 || a->dim <= 0 || a->rot_dim < 0 || a->rot_dim % 2 || a->vdim <= 0 || a->kv_rank <= 0)
    return fail(TLHIP_EINVAL, "%s: bad sizes", who);
  if (a->planes != 1 && a->planes != 3) return fail(TLHIP_EINVAL, "%s: one or three planes", who);
  if (!a->uk || !a->uv || !a->kv_norm || !a->keys || !a->values || (a->rot_dim && !a->angles) || !aligned16(a->uk) || !aligned16(a->uv) ||
      !aligned16(a->keys) || !aligned16(a->values))
    return fail(TLHIP_EINVAL, "%s: null or misaligned operand", who);
  if (a->capacity <= 0 || a->capacity % 32) return fail(TLHIP_EINVAL, "%s: the cache holds whole tiles of 32 keys", who);
  if (a->heads > 4096 || a->dim > 1024 || a->vdim > 4096 || a->kv_rank > 1024 || a->rot_dim > 1024 || a->capacity > (1 << 26))
    return fail(TLHIP_EUNSUPPORTED, "%s: size beyond what the kernels hold", who);
  return TLHIP_OK;
}

// Splits of the keys. A decode step's plan does not depend on the position (it may be on the device).
static int splits(const tlhip_latent_attn* a, int64_t T, int64_t pos0) {
  const int cus = ctx().cus > 0 ? ctx().cus : 256;
  const int64_t keys = a->planes == 1 ? 64 : 32;     // of a block at a time
  const int64_t rts = (T * a->heads + 31) / 32, runs = ((T == 1 ? a->capacity : pos0 + T) + keys - 1) / keys;
  int64_t S = T == 1 ? kMaxSplits : (cus + rts - 1) / rts;
  if (T == 1) S = std::max<int64_t>(1, std::min<int64_t>(S, 2 * cus / rts));
  return (int)std::max<int64_t>(1, std::min<int64_t>({S, runs, kMaxSplits}));
}

typedef void (*attend_fn)(const tlhip_latent_attn, const uint16_t*, float*, int, int, const uint32_t*, int, int);
template <int KS>
static attend_fn pick_values(int nl) {
  return nl <= 1 ? latent_attend_kernel<KS, 1> : nl <= 2 ? latent_attend_kernel<KS, 2> : latent_attend_kernel<KS, 4>;
}
static attend_fn pick_attend(const Dims& d) {
  const int ks = (d.DS + 3) / 4, nl = (d.LT + 7) / 8;
  return ks <= 3 ? pick_values<3>(nl) : ks <= 5 ? pick_values<5>(nl) : ks <= 9 ? pick_values<9>(nl) : ks <= 17 ? pick_values<17>(nl) : nullptr;
}
static attend_fn pick_attend_exact(const Dims& d) {
  const int nl = (d.LT + 3) / 4;
  return nl <= 1 ? latent_attend_exact_kernel<1, 3, 3> : nl <= 2 ? latent_attend_exact_kernel<2, 3, 3>
                       : nl <= 4 ? latent_attend_exact_kernel<4, 3, 3> : latent_attend_exact_kernel<8, 3, 3>;
}

template <int NC, int NQ>
static int launch(const float* u, int64_t ldu, const float* q, int64_t ldq, float* y, int64_t ldy, const tlhip_latent_attn& a, int T,
                  int pos0, const uint32_t* d_pos) {
  constexpr bool kExact = NC == 3;
  Context& c = ctx();
  const Dims d = dims_of(a);
  const int rts = (T * d.H + 31) / 32, rows = rts * 32, S = splits(&a, T, pos0), LV = 32 * d.LT;
  const size_t n_q = (size_t)rts * NQ * d.DS * 512 * sizeof(uint16_t), n_p = (size_t)S * rows * (LV + 2) * sizeof(float);
  char* s = static_cast<char*>(scratch(n_q + n_p));
  if (!s) return fail(TLHIP_ENOMEM, "tlhip_latent_attn: no scratch");
  uint16_t* qimg = reinterpret_cast<uint16_t*>(s);
  float* part = reinterpret_cast<float*>(s + n_q);
  const auto allow = [&](const void* fn, size_t lds) {
    if (lds > (size_t)c.lds_per_cu) return fail(TLHIP_EUNSUPPORTED, "tlhip_latent_attn: not enough LDS");
    if (lds <= 48 * 1024) return (int)TLHIP_OK;
    const hipError_t e = hipFuncSetAttribute(fn, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    return e == hipSuccess ? (int)TLHIP_OK : hip_fail(e, "hipFuncSetAttribute(LDS)");
  };
  // plan everything, then launch
  const int TQ = T == 1 ? 1 : 4, tiles = (T + TQ - 1) / TQ;
  const size_t lqm = (size_t)((d.D + 15) / 16) * 4096, lom = (size_t)d.LT * 4096 + (size_t)32 * S * sizeof(float);
  const bool q_mfma = !kExact && T > 1 && lqm <= 128 * 1024, o_mfma = !kExact && T > 1 && lom <= (size_t)c.lds_per_cu;
  const int slices = q_mfma ? (d.L + kSliceDims - 1) / kSliceDims : (d.DS * 16 + kSliceDims - 1) / kSliceDims;
  const bool q_vec = ldq % 4 == 0 && (d.D + d.R) % 4 == 0 && aligned16(q);
  const bool o_vec = ldy % 4 == 0 && a.y_off % 4 == 0 && d.V % 4 == 0 && aligned16(y) &&
                     (a.gate_off < 0 || (ldu % 4 == 0 && a.gate_off % 4 == 0 && aligned16(u)));
  const size_t lq = q_mfma ? lqm : (size_t)(TQ * d.D + 16 * 16 * 8) * sizeof(float);
  auto fq = TQ == 1 ? latent_query_kernel<1, NC, NQ> : latent_query_kernel<4, NC, NQ>;
  auto fqm = q_vec ? latent_query_mfma_kernel<true> : latent_query_mfma_kernel<false>;
  if (int rc = allow(q_mfma ? reinterpret_cast<const void*>(fqm) : reinterpret_cast<const void*>(fq), lq)) return rc;
  const attend_fn fa = kExact ? pick_attend_exact(d) : pick_attend(d);
  if (!fa) return fail(TLHIP_EUNSUPPORTED, "tlhip_latent_attn: latent and rotated dims beyond what the kernel holds");
  const size_t la = kExact ? (size_t)NQ * d.DS * 1024 + 2 * 16 * 1024 : 0;
  if (int rc = allow(reinterpret_cast<const void*>(fa), la)) return rc;
  const int oslices = (d.V + kOutRows - 1) / kOutRows, ont = TQ == 1 ? 1024 : 256;
  const size_t lo = o_mfma ? lom : (size_t)TQ * (out_groups(ont, TQ, LV) * LV + S) * sizeof(float);
  auto fo = TQ == 1 ? latent_out_kernel<1, 1024> : latent_out_kernel<4, 256>;
  auto fom = o_vec ? latent_out_mfma_kernel<true> : latent_out_mfma_kernel<false>;
  if (int rc = allow(o_mfma ? reinterpret_cast<const void*>(fom) : reinterpret_cast<const void*>(fo), lo)) return rc;

  if (q_mfma) {
    const int64_t items = (int64_t)T * d.H * (d.R / 2 + d.DS * 16 - d.L - d.R), work = (int64_t)slices * d.H * ((T + kQTok - 1) / kQTok);
    const int tail = (int)((items + 255) / 256);
    hipLaunchKernelGGL(fqm, dim3((unsigned)(work + tail + T)), dim3(256), lq, c.stream, u, ldu, q, ldq, a, qimg, T, pos0, slices, tail);
  } else {
    hipLaunchKernelGGL(fq, dim3((unsigned)(slices * d.H * tiles + T)), dim3(256), lq, c.stream, u, ldu, q, ldq, a, qimg, T, pos0, d_pos, slices);
  }
  hipLaunchKernelGGL(fa, dim3((unsigned)(rts * S)), dim3(kExact ? 256 : 512), la, c.stream, a, qimg, part, T, pos0, d_pos, S, rows);
  if (o_mfma)
    hipLaunchKernelGGL(fom, dim3((unsigned)(d.H * ((T + 31) / 32))), dim3(256), lo, c.stream, u, ldu, y, ldy, a, part, T, S, rows);
  else
    hipLaunchKernelGGL(fo, dim3((unsigned)(oslices * d.H * tiles)), dim3((unsigned)ont), lo, c.stream, u, ldu, y, ldy, a, part, T, S, rows, oslices);
  TLHIP_CHECK_LAUNCH(TLHIP_C_LATENT_ATTN);
}

}  // namespace latent
}  // namespace tlhip

using namespace tlhip;

extern "C" {

int64_t tlhip_latent_cache_bytes(int64_t capacity, int64_t kv_rank, int64_t rot_dim, int64_t planes, int values) {
  if (capacity <= 0 || kv_rank <= 0 || rot_dim < 0 || planes <= 0) return 0;
  const int64_t tiles = (capacity + 31) / 32;
  return tiles * planes * (values ? (kv_rank + 31) / 32 * 2048 : (kv_rank + rot_dim + 15) / 16 * 1024);
}

int tlhip_latent_attn_run(const void* u, int64_t ldu, const void* q, int64_t ldq, void* y, int64_t ldy, const tlhip_latent_attn* a,
                          int64_t T, int64_t pos0, const void* d_pos) {
  TLHIP_REQUIRE_READY();
  if (!u || !q || !y || ldu <= 0 || ldq <= 0 || ldy <= 0) return fail(TLHIP_EINVAL, "tlhip_latent_attn_run: bad operands");
  if (int rc = latent::check(a, "tlhip_latent_attn_run")) return rc;
  if (T <= 0 || T > 65535 || pos0 < 0 || pos0 + T > a->capacity || (d_pos && T != 1))
    return fail(TLHIP_EINVAL, "tlhip_latent_attn_run: bad chunk, or past the cache's capacity");
  const float *pu = static_cast<const float*>(u), *pq = static_cast<const float*>(q);
  float* py = static_cast<float*>(y);
  const uint32_t* dp = static_cast<const uint32_t*>(d_pos);
  return a->planes == 1 ? latent::launch<1, 2>(pu, ldu, pq, ldq, py, ldy, *a, (int)T, (int)pos0, dp)
                        : latent::launch<3, 3>(pu, ldu, pq, ldq, py, ldy, *a, (int)T, (int)pos0, dp);
}

}  // extern "C"
