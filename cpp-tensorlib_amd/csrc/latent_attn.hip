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
// Launches: latent_query_kernel (queries into operand images, new cache rows), latent_attend_kernel
// (blocks: query tile x key split, four wavefronts that share a tile's dims), latent_out_kernel (splits
// joined, uv, gate).
#include "common.hpp"

#include <algorithm>

namespace tlhip {
namespace latent {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x16 __attribute__((ext_vector_type(16)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));

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

// ---- attention -----------------------------------------------------------------------------------
// Partials per (split, row): m [S][rows], l [S][rows], acc [S][rows][32 LT].
// Block (query tile, split) of four wavefronts; key tiles split, split + S, ... Scores: every wavefront takes
// each fourth dim step, the four partial sums meet in LDS and every wavefront adds them in the same order.
// Values: wavefront w takes value tiles w, w + 4, ... (NL of them).
template <int NL, int NC, int NQ>
__global__ __launch_bounds__(256) void latent_attend_kernel(const tlhip_latent_attn a, const uint16_t* __restrict__ qimg,
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
#pragma unroll 3
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
// Block (slice of kOutRows value rows, head, TQ <= 4 tokens) of 256 threads.
constexpr int kMaxSplits = 64;
constexpr int kOutRows = 32;
template <int TQ>
__global__ __launch_bounds__(256) void latent_out_kernel(const float* __restrict__ u, int64_t ldu, float* __restrict__ y, int64_t ldy,
                                                         const tlhip_latent_attn a, const float* __restrict__ part, int T, int S,
                                                         int rows, int slices) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const Dims d = dims_of(a);
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int slice = blockIdx.x % slices, h = blockIdx.x / slices % d.H, t0 = blockIdx.x / slices / d.H * TQ;
  const int nt = min(TQ, T - t0), LV = 32 * d.LT, ldv = up8(d.L);
  float* oc = lds;                     // [TQ][LV] normalised sums of latents
  float* w = oc + TQ * LV;             // [TQ][S] the splits' weights
  const size_t R = (size_t)rows;
  const float *pm = part, *pl = part + (size_t)S * R, *pa = pl + (size_t)S * R;
  if (wave < TQ) {                     // a wavefront weighs the (up to 64) splits of one token
    const int row = (t0 + min(wave, nt - 1)) * d.H + h;
    const float m = lane < S ? pm[lane * R + row] : -INFINITY, l = lane < S ? pl[lane * R + row] : 0.f;
    const float f = exp2f(m - wave_max(m)), tot = wave_sum(f * l);
    if (lane < S) w[wave * S + lane] = f / tot;
  }
  __syncthreads();
  for (int i = tid; i < TQ * (LV / 4); i += 256) {
    const int t = i / (LV / 4), e = 4 * (i - t * (LV / 4));
    const float* src = pa + ((size_t)(t0 + min(t, nt - 1)) * d.H + h) * LV + e;
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    for (int s0 = 0; s0 < S; s0 += 8) {
      f32x4 v[8];
#pragma unroll
      for (int k = 0; k < 8; k++) v[k] = *reinterpret_cast<const f32x4*>(src + (size_t)min(s0 + k, S - 1) * R * LV);
#pragma unroll
      for (int k = 0; k < 8; k++)
        if (s0 + k < S) {
          const float f = w[t * S + s0 + k];
          acc += v[k] * f;
        }
    }
    *reinterpret_cast<f32x4*>(oc + t * LV + e) = acc;
  }
  __syncthreads();
  const int v1 = min(d.V, (slice + 1) * kOutRows), n8 = ldv / 8;
  const u32x4* uv = reinterpret_cast<const u32x4*>(static_cast<const uint16_t*>(a.uv)) + (size_t)h * d.V * n8;
  for (int v = slice * kOutRows + wave; v < v1; v += 4) {
    float acc[TQ];
#pragma unroll
    for (int t = 0; t < TQ; t++) acc[t] = 0.f;
    for (int k = lane; k < n8; k += 64) {
      const u32x4 x = uv[(size_t)v * n8 + k];
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
        if (a.gate_off >= 0) o = s / (1.f + expf(-u[(size_t)(t0 + t) * ldu + a.gate_off + h * d.V + v]));
        y[(size_t)(t0 + t) * ldy + a.y_off + h * d.V + v] = o;
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
  const int64_t rts = (T * a->heads + 31) / 32, tiles = T == 1 ? a->capacity / 32 : (pos0 + T + 31) / 32;
  int64_t S = T == 1 ? kMaxSplits : (cus + rts - 1) / rts;
  if (T == 1) S = std::max<int64_t>(1, std::min<int64_t>(S, 2 * cus / rts));
  return (int)std::max<int64_t>(1, std::min<int64_t>({S, tiles, kMaxSplits}));
}

template <int NC, int NQ>
static int launch(const float* u, int64_t ldu, const float* q, int64_t ldq, float* y, int64_t ldy, const tlhip_latent_attn& a, int T,
                  int pos0, const uint32_t* d_pos) {
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
  const int TQ = T == 1 ? 1 : 4, tiles = (T + TQ - 1) / TQ, slices = (d.DS * 16 + kSliceDims - 1) / kSliceDims;
  const size_t lq = (size_t)(TQ * d.D + 16 * 16 * 8) * sizeof(float);
  auto fq = TQ == 1 ? latent_query_kernel<1, NC, NQ> : latent_query_kernel<4, NC, NQ>;
  if (int rc = allow(reinterpret_cast<const void*>(fq), lq)) return rc;
  const size_t la = (size_t)NQ * d.DS * 1024 + 2 * 16 * 1024;
  const int nl = (d.LT + 3) / 4;
  auto fa = nl <= 1 ? latent_attend_kernel<1, NC, NQ> : nl <= 2 ? latent_attend_kernel<2, NC, NQ> : nl <= 4 ? latent_attend_kernel<4, NC, NQ>
                                                                                                    : latent_attend_kernel<8, NC, NQ>;
  if (int rc = allow(reinterpret_cast<const void*>(fa), la)) return rc;
  const int oslices = (d.V + kOutRows - 1) / kOutRows;
  const size_t lo = (size_t)TQ * (LV + S) * sizeof(float);
  auto fo = TQ == 1 ? latent_out_kernel<1> : latent_out_kernel<4>;
  if (int rc = allow(reinterpret_cast<const void*>(fo), lo)) return rc;
  hipLaunchKernelGGL(fq, dim3((unsigned)(slices * d.H * tiles + T)), dim3(256), lq, c.stream, u, ldu, q, ldq, a, qimg, T, pos0, d_pos, slices);
  hipLaunchKernelGGL(fa, dim3((unsigned)(rts * S)), dim3(256), la, c.stream, a, qimg, part, T, pos0, d_pos, S, rows);
  hipLaunchKernelGGL(fo, dim3((unsigned)(oslices * d.H * tiles)), dim3(256), lo, c.stream, u, ldu, y, ldy, a, part, T, S, rows, oslices);
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
