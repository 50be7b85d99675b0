// Prompt chunks of the sliding-window attention whose values are its keys, on the fp32 matrix pipe,
// and the copy of a chunk's keys into the ring.
//
// A block owns one query head and 32 consecutive positions; its NW wavefronts deal the 32-key tiles
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
#include "attn_window.hpp"

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
                            int64_t pos0) {
  TLHIP_REQUIRE_READY();
  if (!y || ldy <= 0) return fail(TLHIP_EINVAL, "tlhip_window_attn_chunk: bad operands");
  if (int rc = check_chunk(u, ldu, T, pos0, at, "tlhip_window_attn_chunk")) return rc;
  const float* pu = static_cast<const float*>(u);
  float* py = static_cast<float*>(y);
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
