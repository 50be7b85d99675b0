// State-space layer with one decay per head and step (Mamba-2): short causal convolution, recurrence,
// skip, gate. Per head h of group g, token t:
//   xbc = silu(conv(x | B | C)),  dt = softplus(dt + bias),  S <- a S + dt B x^T,  a = 2^(decay_h dt),
//   y = (S^T C + skip_h x) silu(z)
// decay_h is the base-2 log of the decay per unit of dt (negative). Everything is f32.
//
// Decode: one block per head (ssm_step_kernel). Prompt chunks in pieces of C tokens, with l_t the sum of
// the log decays since the piece began:
//   y_t = 2^l_t C_t^T S_0 + sum_(s <= t) (C_t . B_s) 2^(l_t - l_s) dt_s x_s
//   S_C = 2^l_C S_0 + sum_s 2^(l_C - l_s) dt_s B_s x_s^T
// every exponent <= 0. Four launches: ssm_conv_kernel (convolution, activation; steps and log decays), ssm_piece_kernel
// (each piece's own part of S_C), ssm_scan_kernel (the state through the pieces, the convolution's new
// tail), ssm_out_kernel (y). Products on the fp32 matrix pipe.
//
// State: two slots by the position's parity (a step reads slot p % 2 and writes the other, so it can be
// repeated), position 0 reads zeros. Convolution inputs: a ring of `taps` rows, position p at p % taps.
#include "common.hpp"

#include <algorithm>

namespace tlhip {

typedef float f32x4 __attribute__((ext_vector_type(4)));
__device__ __forceinline__ f32x4 ssm_mfma(float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }
__device__ __forceinline__ float silu_f(float z) { return z / (1.f + expf(-z)); }
__device__ __forceinline__ float softplus_f(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

struct SsmDims {
  int H, N, G, V, taps, inner, ch;   // ch: channels of the convolution, inner + 2 G N
};
__host__ __device__ inline SsmDims ssm_dims(const tlhip_ssm& a) {
  SsmDims d;
  d.H = (int)a.heads; d.N = (int)a.state; d.G = (int)a.groups; d.V = (int)a.vdim; d.taps = (int)a.taps;
  d.inner = d.H * d.V;
  d.ch = d.inner + 2 * d.G * d.N;
  return d;
}
__host__ __device__ inline int ssm_ld(int V) { return (V + 3) & ~3; }

// sum over the taps of channel c for the token at position p; `now` is the token's own input
__device__ __forceinline__ float conv_step(const tlhip_ssm& a, const SsmDims& d, const float* __restrict__ ring, int p, int c, float now) {
  const float* w = static_cast<const float*>(a.conv_w);
  float s = 0.f;
  for (int j = 0; j < d.taps - 1; j++) {
    const int q = p - (d.taps - 1) + j;
    const float x = ring[(size_t)(max(q, 0) % d.taps) * d.ch + c];
    s = fmaf(w[(size_t)j * d.ch + c], q >= 0 ? x : 0.f, s);
  }
  return fmaf(w[(size_t)(d.taps - 1) * d.ch + c], now, s) + static_cast<const float*>(a.conv_b)[c];
}

// Decode step of one head, 512 threads: a thread owns one float4 column of every ng-th state row.
__global__ __launch_bounds__(512) void ssm_step_kernel(const float* __restrict__ u, float* __restrict__ y, const tlhip_ssm a,
                                                       int pos, const uint32_t* __restrict__ d_pos) {
  extern __shared__ __attribute__((aligned(16))) float ssm_lds[];
  const SsmDims d = ssm_dims(a);
  const int tid = threadIdx.x, h = blockIdx.x, per = d.H / d.G, g = h / per;
  const int p = d_pos ? (int)*d_pos : pos;
  const int ld = ssm_ld(d.V), nv4 = ld >> 2, ng = 512 / nv4, v4 = tid % nv4, ng0 = tid / nv4;
  const bool live = ng0 < ng;
  float* xs = ssm_lds;                 // [ld] convolved x of the head
  float* Bs = xs + ld;                 // [N]
  float* Cs = Bs + d.N;                // [N]
  float* red = Cs + d.N + ((4 - (ld + 2 * d.N) % 4) & 3);   // [ng][ld]
  const size_t slot = (size_t)d.H * d.N * ld;
  const float* src = static_cast<const float*>(a.ssm_state) + (size_t)(p & 1) * slot + (size_t)h * d.N * ld;
  float* dst = static_cast<float*>(a.ssm_state) + (size_t)((p + 1) & 1) * slot + (size_t)h * d.N * ld;
  constexpr int PRE = 8;               // rows of this thread requested up front
  float4 st[PRE];
#pragma unroll
  for (int i = 0; i < PRE; i++) {
    const int n = ng0 + i * ng;
    st[i] = live && p > 0 && n < d.N ? *reinterpret_cast<const float4*>(src + (size_t)n * ld + 4 * v4) : make_float4(0.f, 0.f, 0.f, 0.f);
  }
  float* ring = static_cast<float*>(a.conv_state);
  const float dt = softplus_f(u[a.dt_off + h] + static_cast<const float*>(a.dt_bias)[h]);
  const float w = exp2f(static_cast<const float*>(a.decay)[h] * dt);
  // this head's x and its group's B and C; the input row is kept for the coming tokens (B, C: by the group's first head)
  for (int i = tid; i < ld + 2 * d.N; i += 512) {
    int c;
    bool keep = true;
    if (i < ld) c = i < d.V ? h * d.V + i : -1;
    else {
      const int n = i - ld;
      c = d.inner + (n < d.N ? g * d.N + n : (d.G + g) * d.N + n - d.N);
      keep = h == g * per;
    }
    float v = 0.f;
    if (c >= 0) {
      const float now = u[a.x_off + c];
      v = silu_f(conv_step(a, d, ring, p, c, now));
      if (keep) ring[(size_t)(p % d.taps) * d.ch + c] = now;
    }
    ssm_lds[i] = v;
  }
  __syncthreads();
  if (live) {
    float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
    const float x0 = dt * xs[4 * v4], x1 = dt * xs[4 * v4 + 1], x2 = dt * xs[4 * v4 + 2], x3 = dt * xs[4 * v4 + 3];
    const auto row = [&](int n, float4 s) {
      const float b = Bs[n], c = Cs[n];
      s.x = fmaf(w, s.x, b * x0); s.y = fmaf(w, s.y, b * x1); s.z = fmaf(w, s.z, b * x2); s.w = fmaf(w, s.w, b * x3);
      *reinterpret_cast<float4*>(dst + (size_t)n * ld + 4 * v4) = s;
      o.x = fmaf(c, s.x, o.x); o.y = fmaf(c, s.y, o.y); o.z = fmaf(c, s.z, o.z); o.w = fmaf(c, s.w, o.w);
    };
#pragma unroll
    for (int i = 0; i < PRE; i++)
      if (ng0 + i * ng < d.N) row(ng0 + i * ng, st[i]);
    for (int n = ng0 + PRE * ng; n < d.N; n += ng)
      row(n, p > 0 ? *reinterpret_cast<const float4*>(src + (size_t)n * ld + 4 * v4) : make_float4(0.f, 0.f, 0.f, 0.f));
    *reinterpret_cast<float4*>(red + ng0 * ld + 4 * v4) = o;
  }
  __syncthreads();
  for (int v = tid; v < d.V; v += 512) {
    float t = 0.f;
    for (int k = 0; k < ng; k++) t += red[k * ld + v];
    t = fmaf(static_cast<const float*>(a.skip)[h], xs[v], t);
    y[a.y_off + h * d.V + v] = t * silu_f(u[a.z_off + h * d.V + v]);
  }
}
static size_t ssm_step_lds(const tlhip_ssm& a) {
  const int ld = ssm_ld((int)a.vdim), ng = 512 / (ld >> 2);
  return (size_t)(ld + 2 * (int)a.state + 4 + ng * ld) * sizeof(float);
}

// ---- prompt chunks -------------------------------------------------------------------------------
// Scratch of a call: convolved rows [T][xw] = [x: H x Vp | B: G x Np | C: G x Np] (Vp, Np: V and N rounded up
// to 16, zeros between), dt [T][H], log decays summed since the piece began [T][H], and per piece and head
// the state ahead of it [Np][Vp].
struct SsmBuf {
  float *xbc, *dt, *lsum, *st;
  int C, np, Vp, Np, xw;
};

constexpr int kConvTok = 16;         // tokens of one block of ssm_conv_kernel

// dt and the log decays summed along each piece: a wavefront owns a head and a piece, a lane a token.
__device__ __forceinline__ void ssm_steps(const float* __restrict__ u, int64_t ldu, const tlhip_ssm& a, int T, const SsmBuf& b, int i) {
  const int H = (int)a.heads;
  if (i >= H * b.np) return;
  const int lane = threadIdx.x & 63, h = i % H, t = i / H * b.C + lane;
  const bool live = lane < b.C && t < T;
  const float dt = softplus_f(u[(size_t)min(t, T - 1) * ldu + a.dt_off + h] + static_cast<const float*>(a.dt_bias)[h]);
  float l = live ? static_cast<const float*>(a.decay)[h] * dt : 0.f;
#pragma unroll
  for (int k = 1; k < 64; k *= 2) {
    const float o = __shfl_up(l, k, kWave);
    if (lane >= k) l += o;
  }
  if (live) {
    b.dt[(size_t)t * H + h] = dt;
    b.lsum[(size_t)t * H + h] = l;
  }
}

// Grid (columns of xbc / 256, then steps; token tiles). TAPS 0: any number of taps.
template <int TAPS>
__global__ __launch_bounds__(256) void ssm_conv_kernel(const float* __restrict__ u, int64_t ldu, const tlhip_ssm a, int T, int pos0,
                                                       const SsmBuf b, int cols) {
  if ((int)blockIdx.x >= cols) {
    ssm_steps(u, ldu, a, T, b, (((int)blockIdx.x - cols) * (int)gridDim.y + (int)blockIdx.y) * 4 + ((int)threadIdx.x >> 6));
    return;
  }
  const SsmDims d = ssm_dims(a);
  const int j = blockIdx.x * 256 + threadIdx.x, t0 = blockIdx.y * kConvTok, t1 = min(T, t0 + kConvTok);
  if (j >= b.xw) return;
  int c = -1;
  const int xn = d.H * b.Vp, gn = d.G * b.Np;
  if (j < xn) {
    const int v = j % b.Vp;
    if (v < d.V) c = j / b.Vp * d.V + v;
  } else {
    const int k = (j - xn) % gn, n = k % b.Np;
    if (n < d.N) c = d.inner + ((j - xn) / gn * d.G + k / b.Np) * d.N + n;
  }
  float* o = b.xbc + j;
  if (c < 0) {
    for (int t = t0; t < t1; t++) o[(size_t)t * b.xw] = 0.f;
    return;
  }
  const float* w = static_cast<const float*>(a.conv_w) + c;
  const float* ring = static_cast<const float*>(a.conv_state) + c;
  const float bias = static_cast<const float*>(a.conv_b)[c];
  const float* x = u + a.x_off + c;
  const auto input = [&](int t) -> float {          // token t of the chunk, or one of those before it
    if (t >= 0) return x[(size_t)t * ldu];
    const int p = pos0 + t;
    return p >= 0 ? ring[(size_t)(p % d.taps) * d.ch] : 0.f;
  };
  if constexpr (TAPS > 0) {
    float wt[TAPS], in[TAPS - 1 + kConvTok];
#pragma unroll
    for (int k = 0; k < TAPS; k++) wt[k] = w[(size_t)k * d.ch];
#pragma unroll
    for (int k = 0; k < TAPS - 1; k++) in[k] = input(t0 - (TAPS - 1) + k);
#pragma unroll
    for (int k = 0; k < kConvTok; k++) in[TAPS - 1 + k] = x[(size_t)min(t0 + k, T - 1) * ldu];
#pragma unroll
    for (int k = 0; k < kConvTok; k++) {
      float s = 0.f;
#pragma unroll
      for (int i = 0; i < TAPS; i++) s = fmaf(wt[i], in[k + i], s);
      if (t0 + k < t1) o[(size_t)(t0 + k) * b.xw] = silu_f(s + bias);
    }
  } else {
    for (int t = t0; t < t1; t++) {
      float s = 0.f;
      for (int i = 0; i < d.taps; i++) s = fmaf(w[(size_t)i * d.ch], input(t - (d.taps - 1) + i), s);
      o[(size_t)t * b.xw] = silu_f(s + bias);
    }
  }
}

// Rows [0, C) x cols [0, n) of src into LDS rows of `ld`, zeros past `rows`; n a multiple of 4.
__device__ __forceinline__ void ssm_tile(float* __restrict__ dst, int ld, const float* __restrict__ src, int64_t lds_src, int C, int n,
                                         int rows, int tid, int nt) {
  const int n4 = n >> 2;
  for (int i = tid; i < C * n4; i += nt) {
    const int t = i / n4, c = 4 * (i - t * n4);
    f32x4 v = *reinterpret_cast<const f32x4*>(src + (size_t)min(t, rows - 1) * lds_src + c);
    if (t >= rows) v = f32x4{0.f, 0.f, 0.f, 0.f};
    *reinterpret_cast<f32x4*>(dst + t * ld + c) = v;
  }
}

// Block (piece, head) of 256 threads: sum over s of 2^(l_C - l_s) dt_s B_s x_s^T.
template <int C>
__global__ __launch_bounds__(256) void ssm_piece_kernel(const tlhip_ssm a, int T, const SsmBuf b) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const SsmDims d = ssm_dims(a);
  const int tid = threadIdx.x, lane = tid & 63, l15 = lane & 15, lg = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int piece = blockIdx.x, h = blockIdx.y, g = h / (d.H / d.G), t0 = piece * C, nt = min(C, T - t0);
  const int BS = b.Np + 4, XS = b.Vp + 4;
  float* B = lds;                      // [C][BS]
  float* X = B + C * BS;               // [C][XS]
  float* W = X + C * XS;               // [C]
  const float* row = b.xbc + (size_t)t0 * b.xw;
  ssm_tile(B, BS, row + d.H * b.Vp + g * b.Np, b.xw, C, b.Np, nt, tid, 256);
  ssm_tile(X, XS, row + h * b.Vp, b.xw, C, b.Vp, nt, tid, 256);
  if (tid < C) {
    const int t = t0 + min(tid, nt - 1);
    const float lc = b.lsum[(size_t)(t0 + nt - 1) * d.H + h];
    W[tid] = tid < nt ? exp2f(lc - b.lsum[(size_t)t * d.H + h]) * b.dt[(size_t)t * d.H + h] : 0.f;
  }
  __syncthreads();
  const int nvt = b.Vp / 16, groups = (nvt + 3) / 4;
  float* st = b.st + ((size_t)h * b.np + piece) * b.Np * b.Vp;
  for (int tile = wave; tile < (b.Np / 16) * groups; tile += 4) {
    const int n = 16 * (tile / groups) + l15, vt = 4 * (tile % groups), n4 = min(4, nvt - vt);
    f32x4 acc[4];
#pragma unroll
    for (int k = 0; k < 4; k++) acc[k] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int s0 = 0; s0 < C; s0 += 4) {
      const int s = s0 + lg;
      const float bw = B[s * BS + n] * W[s];
#pragma unroll
      for (int k = 0; k < 4; k++) acc[k] = ssm_mfma(bw, X[s * XS + 16 * (vt + min(k, n4 - 1)) + l15], acc[k]);
    }
#pragma unroll
    for (int k = 0; k < 4; k++)
      if (k < n4)
#pragma unroll
        for (int i = 0; i < 4; i++) st[(size_t)(n - l15 + 4 * lg + i) * b.Vp + 16 * (vt + k) + l15] = acc[k][i];
  }
}

// The state through the pieces: st[piece] becomes the state ahead of the piece, the last one goes to its slot;
// a thread owns four value columns of one row. The blocks past those keep the convolution's newest inputs.
__global__ __launch_bounds__(256) void ssm_scan_kernel(const float* __restrict__ u, int64_t ldu, const tlhip_ssm a, int T, int pos0,
                                                       const SsmBuf b, int scan_blocks) {
  const SsmDims d = ssm_dims(a);
  if ((int)blockIdx.x >= scan_blocks) {
    const int c = ((int)blockIdx.x - scan_blocks) * 256 + threadIdx.x;
    if (c >= d.ch) return;
    float* ring = static_cast<float*>(a.conv_state);
    for (int t = max(0, T - d.taps); t < T; t++) ring[(size_t)((pos0 + t) % d.taps) * d.ch + c] = u[(size_t)t * ldu + a.x_off + c];
    return;
  }
  const int ld = ssm_ld(d.V), nv4 = b.Vp / 4;
  const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= (size_t)d.H * b.Np * nv4) return;
  const int v = 4 * (int)(i % nv4), n = (int)(i / nv4 % b.Np), h = (int)(i / nv4 / b.Np);
  const size_t slot = (size_t)d.H * d.N * ld, at = ((size_t)h * d.N + n) * ld + v;
  const bool kept = n < d.N && v < ld;
  float* state = static_cast<float*>(a.ssm_state);
  float4 s = make_float4(0.f, 0.f, 0.f, 0.f);
  if (kept && pos0 > 0) s = *reinterpret_cast<const float4*>(state + (size_t)(pos0 & 1) * slot + at);
  constexpr int U = 8;                 // pieces requested at once
  for (int p0 = 0; p0 < b.np; p0 += U) {
    float4 t[U];
    float w[U];
#pragma unroll
    for (int k = 0; k < U; k++) {
      const int p = min(p0 + k, b.np - 1);
      t[k] = *reinterpret_cast<const float4*>(b.st + (((size_t)h * b.np + p) * b.Np + n) * b.Vp + v);
      w[k] = b.lsum[(size_t)(min(T, (p + 1) * b.C) - 1) * d.H + h];
    }
#pragma unroll
    for (int k = 0; k < U; k++)
      if (p0 + k < b.np) {
        const float f = exp2f(w[k]);
        *reinterpret_cast<float4*>(b.st + (((size_t)h * b.np + p0 + k) * b.Np + n) * b.Vp + v) = s;
        s.x = fmaf(f, s.x, t[k].x); s.y = fmaf(f, s.y, t[k].y); s.z = fmaf(f, s.z, t[k].z); s.w = fmaf(f, s.w, t[k].w);
      }
  }
  if (kept) *reinterpret_cast<float4*>(state + (size_t)((pos0 + T) & 1) * slot + at) = s;
}

// Block (piece, head) of 512 threads: C_t . B_s with the head's decays and steps, then both terms of y, skip and gate.
// What is needed last - x and the state ahead of the piece - is requested first.
template <int C>
__global__ __launch_bounds__(512) __attribute__((amdgpu_waves_per_eu(4))) void ssm_out_kernel(const float* __restrict__ u, int64_t ldu, float* __restrict__ y, int64_t ldy,
                                                      const tlhip_ssm a, int T, const SsmBuf b) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  constexpr int NB = C / 16, AS = C + 4, NW = 8, HALF = NB > 1 ? NB / 2 : 1;
  constexpr int TILES = NB * (NB + 1) / 2, TW = (TILES + NW - 1) / NW;   // tiles of C . B, of a wavefront
  const SsmDims d = ssm_dims(a);
  const int tid = threadIdx.x, lane = tid & 63, l15 = lane & 15, lg = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int piece = blockIdx.x, h = blockIdx.y, g = h / (d.H / d.G);
  const int t0 = piece * C, nt = min(C, T - t0), BS = b.Np + 4, XS = b.Vp + 4;
  float* Cm = lds;                     // [C][BS]
  float* B = Cm + C * BS;              // [C][BS], then
  float* M = B;                        // [C][AS] C_t . B_s 2^(l_t - l_s) dt_s, s <= t, and
  float* X = M + C * AS;               // [C][XS] x of the head
  float* L = B + max(C * BS, C * (AS + XS));   // [C] log decay sums, [C] steps
  float* D = L + C;
  const float* row = b.xbc + (size_t)t0 * b.xw;
  const float* st = b.st + ((size_t)h * b.np + piece) * b.Np * b.Vp;
  const int nvt = b.Vp / 16, v4 = b.Vp >> 2, items = nvt * (NB > 1 ? 2 : 1);
  constexpr int XR = 2;
  f32x4 xr[XR];
#pragma unroll
  for (int k = 0; k < XR; k++) {
    const int i = min(tid + 512 * k, C * v4 - 1), t = i / v4;
    xr[k] = *reinterpret_cast<const f32x4*>(row + (size_t)min(t, nt - 1) * b.xw + h * b.Vp + 4 * (i - t * v4));
  }
  float sv[4][4];                      // state rows n0 .. n0 + 63 of an item's columns
  const auto load_state = [&](int item, int n0) {
    const int v = 16 * (item % nvt) + l15;
#pragma unroll
    for (int k = 0; k < 4; k++)
#pragma unroll
      for (int e = 0; e < 4; e++) sv[k][e] = st[(size_t)(min(n0 + 16 * k, b.Np - 16) + 4 * lg + e) * b.Vp + v];
  };
  load_state(min(wave, items - 1), 0);
  ssm_tile(Cm, BS, row + d.H * b.Vp + (d.G + g) * b.Np, b.xw, C, b.Np, nt, tid, 512);
  ssm_tile(B, BS, row + d.H * b.Vp + g * b.Np, b.xw, C, b.Np, nt, tid, 512);
  if (tid < C) {
    const int t = t0 + min(tid, nt - 1);
    L[tid] = b.lsum[(size_t)t * d.H + h];
    D[tid] = tid < nt ? b.dt[(size_t)t * d.H + h] : 0.f;
  }
  __syncthreads();
  f32x4 cb[TW];
#pragma unroll
  for (int w = 0; w < TW; w++) {
    cb[w] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (wave + NW * w >= TILES) continue;
    int i = 0, j = wave + NW * w;
    while (j > i) { i++; j -= i; }
    for (int n0 = 0; n0 < b.Np; n0 += 16) {
      const f32x4 cf = *reinterpret_cast<const f32x4*>(Cm + (16 * i + l15) * BS + n0 + 4 * lg);
      const f32x4 bf = *reinterpret_cast<const f32x4*>(B + (16 * j + l15) * BS + n0 + 4 * lg);
#pragma unroll
      for (int k = 0; k < 4; k++) cb[w] = ssm_mfma(cf[k], bf[k], cb[w]);
    }
  }
  __syncthreads();                     // B has been read
#pragma unroll
  for (int w = 0; w < TW; w++) {
    if (wave + NW * w >= TILES) continue;
    int i = 0, j = wave + NW * w;
    while (j > i) { i++; j -= i; }
    const int s = 16 * j + l15;
#pragma unroll
    for (int k = 0; k < 4; k++) {
      const int t = 16 * i + 4 * lg + k;
      M[t * AS + s] = s <= t ? cb[w][k] * exp2f(L[t] - L[s]) * D[s] : 0.f;
    }
  }
  for (int i = tid, k = 0; i < C * v4; i += 512, k++) {
    const int t = i / v4, c = 4 * (i - t * v4);
    f32x4 v;
    if (k == 0) v = xr[0];
    else if (k == 1) v = xr[1];
    else v = *reinterpret_cast<const f32x4*>(row + (size_t)min(t, nt - 1) * b.xw + h * b.Vp + c);
    if (t >= nt) v = f32x4{0.f, 0.f, 0.f, 0.f};
    *reinterpret_cast<f32x4*>(X + t * XS + c) = v;
  }
  __syncthreads();
  const float skip = static_cast<const float*>(a.skip)[h];
  // an item: 16 value columns and half of the row blocks, k and NB - 1 - k, which balances the triangle
  for (int item = wave; item < items; item += NW) {
    const int v0 = 16 * (item % nvt), half = item / nvt;
    f32x4 acc[2];
    float z[2][4];
    int blk[2];
#pragma unroll
    for (int r = 0; r < 2; r++) {
      blk[r] = NB == 1 ? 0 : NB == 2 ? half : r ? NB - 1 - half : half;
      acc[r] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (r >= HALF) continue;
#pragma unroll
      for (int k = 0; k < 4; k++)
        z[r][k] = u[(size_t)(t0 + min(16 * blk[r] + 4 * lg + k, nt - 1)) * ldu + a.z_off + h * d.V + min(v0 + l15, d.V - 1)];
    }
    if (item != wave) load_state(item, 0);
    for (int n0 = 0; n0 < b.Np; n0 += 64) {
      if (n0 > 0) load_state(item, n0);
#pragma unroll
      for (int k = 0; k < 4; k++) {
        const int n = n0 + 16 * k;
        if (n >= b.Np) continue;
#pragma unroll
        for (int r = 0; r < HALF; r++) {
          const f32x4 cf = *reinterpret_cast<const f32x4*>(Cm + (16 * blk[r] + l15) * BS + n + 4 * lg);
#pragma unroll
          for (int e = 0; e < 4; e++) acc[r] = ssm_mfma(cf[e], sv[k][e], acc[r]);
        }
      }
    }
#pragma unroll
    for (int r = 0; r < HALF; r++) {
      const int i = blk[r];
#pragma unroll
      for (int k = 0; k < 4; k++) acc[r][k] *= exp2f(L[16 * i + 4 * lg + k]);
      for (int j = 0; j <= i; j++) {
        const f32x4 m = *reinterpret_cast<const f32x4*>(M + (16 * i + l15) * AS + 16 * j + 4 * lg);
#pragma unroll
        for (int e = 0; e < 4; e++) acc[r] = ssm_mfma(m[e], X[(16 * j + 4 * lg + e) * XS + v0 + l15], acc[r]);
      }
      const int v = v0 + l15;
#pragma unroll
      for (int k = 0; k < 4; k++) {
        const int t = 16 * i + 4 * lg + k;
        if (t < nt && v < d.V) y[(size_t)(t0 + t) * ldy + a.y_off + h * d.V + v] = fmaf(skip, X[t * XS + v], acc[r][k]) * silu_f(z[r][k]);
      }
    }
  }
}

static size_t ssm_piece_lds(int C, int Np, int Vp) { return (size_t)(C * (Np + 4) + C * (Vp + 4) + C) * sizeof(float); }
static size_t ssm_out_lds(int C, int Np, int Vp) {
  return (size_t)(C * (Np + 4) + std::max(C * (Np + 4), C * (C + 4 + Vp + 4)) + 2 * C) * sizeof(float);
}

static int check_ssm(const tlhip_ssm* a, const char* who) {
  if (!a || a->heads <= 0 || a->state <= 0 || a->groups <= 0 || a->heads % a->groups || a->vdim <= 0 || a->taps <= 0)
    return fail(TLHIP_EINVAL, "%s: bad sizes", who);
  if (!a->conv_w || !a->conv_b || !a->dt_bias || !a->decay || !a->skip || !a->conv_state || !a->ssm_state || !aligned16(a->ssm_state))
    return fail(TLHIP_EINVAL, "%s: null or misaligned operand", who);
  if (a->heads > 65535 || a->vdim > 1024 || a->state > 512 || a->taps > 64)
    return fail(TLHIP_EUNSUPPORTED, "%s: heads beyond a state of 512 x 1024, or more than 64 taps", who);
  return TLHIP_OK;
}

}  // namespace tlhip

using namespace tlhip;

extern "C" {

int64_t tlhip_ssm_state_bytes(int64_t heads, int64_t state, int64_t vdim) {
  return 2 * heads * state * ssm_ld((int)vdim) * (int64_t)sizeof(float);
}
int64_t tlhip_ssm_conv_bytes(int64_t heads, int64_t state, int64_t groups, int64_t vdim, int64_t taps) {
  return taps * (heads * vdim + 2 * groups * state) * (int64_t)sizeof(float);
}

int tlhip_ssm_step(const void* u, void* y, const tlhip_ssm* a, int64_t pos, const void* d_pos) {
  TLHIP_REQUIRE_READY();
  if (!u || !y || pos < 0 || pos > (1 << 30)) return fail(TLHIP_EINVAL, "tlhip_ssm_step: bad operands");
  if (int rc = check_ssm(a, "tlhip_ssm_step")) return rc;
  Context& c = ctx();
  const size_t lds = ssm_step_lds(*a);
  if (lds > (size_t)c.lds_per_cu) return fail(TLHIP_EUNSUPPORTED, "tlhip_ssm_step: not enough LDS");
  hipLaunchKernelGGL(ssm_step_kernel, dim3((unsigned)a->heads), dim3(512), lds, c.stream, static_cast<const float*>(u),
                     static_cast<float*>(y), *a, (int)pos, static_cast<const uint32_t*>(d_pos));
  TLHIP_CHECK_LAUNCH(TLHIP_C_SSM);
}

int tlhip_ssm_chunk(const void* u, int64_t ldu, void* y, int64_t ldy, const tlhip_ssm* a, int64_t T, int64_t pos0) {
  TLHIP_REQUIRE_READY();
  if (!u || !y || ldu <= 0 || ldy <= 0) return fail(TLHIP_EINVAL, "tlhip_ssm_chunk: bad operands");
  if (T <= 0 || T > (1 << 20) || pos0 < 0 || pos0 + T > (1 << 30)) return fail(TLHIP_EINVAL, "tlhip_ssm_chunk: bad chunk");
  if (int rc = check_ssm(a, "tlhip_ssm_chunk")) return rc;
  Context& c = ctx();
  SsmBuf b{};
  b.Vp = (int)(a->vdim + 15) / 16 * 16;
  b.Np = (int)(a->state + 15) / 16 * 16;
  b.xw = (int)a->heads * b.Vp + 2 * (int)a->groups * b.Np;
  b.C = 64;
  while (b.C > 16 && (std::max(ssm_out_lds(b.C, b.Np, b.Vp), ssm_piece_lds(b.C, b.Np, b.Vp)) > (size_t)c.lds_per_cu || b.C / 2 >= T)) b.C /= 2;
  const size_t lds1 = ssm_piece_lds(b.C, b.Np, b.Vp), lds2 = ssm_out_lds(b.C, b.Np, b.Vp);
  if (std::max(lds1, lds2) > (size_t)c.lds_per_cu) return fail(TLHIP_EUNSUPPORTED, "tlhip_ssm_chunk: head too large for LDS");
  b.np = (int)((T + b.C - 1) / b.C);
  const size_t n_x = ((size_t)T * b.xw + 3) & ~(size_t)3, n_d = ((size_t)T * a->heads + 3) & ~(size_t)3,
               n_st = (size_t)a->heads * b.np * b.Np * b.Vp;
  float* s = static_cast<float*>(scratch((n_x + 2 * n_d + n_st) * sizeof(float)));
  if (!s) return fail(TLHIP_ENOMEM, "tlhip_ssm_chunk: no scratch");
  b.xbc = s;
  b.st = b.xbc + n_x;
  b.dt = b.st + n_st;
  b.lsum = b.dt + n_d;
  const float* pu = static_cast<const float*>(u);
  const unsigned tt = (unsigned)((T + kConvTok - 1) / kConvTok);
  if (tt > 65535) return fail(TLHIP_EUNSUPPORTED, "tlhip_ssm_chunk: chunk too long");
  auto conv = a->taps == 4 ? ssm_conv_kernel<4> : a->taps == 3 ? ssm_conv_kernel<3> : a->taps == 2 ? ssm_conv_kernel<2> : ssm_conv_kernel<0>;
  const int cols = (b.xw + 255) / 256, steps = (int)(((a->heads * b.np + 3) / 4 + tt - 1) / tt);
  hipLaunchKernelGGL(conv, dim3((unsigned)(cols + steps), tt), dim3(256), 0, c.stream, pu, ldu, *a, (int)T, (int)pos0, b, cols);
  auto piece = b.C == 64 ? ssm_piece_kernel<64> : b.C == 32 ? ssm_piece_kernel<32> : ssm_piece_kernel<16>;
  hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(piece), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds1);
  if (e != hipSuccess) return hip_fail(e, "hipFuncSetAttribute(LDS)");
  hipLaunchKernelGGL(piece, dim3((unsigned)b.np, (unsigned)a->heads), dim3(256), lds1, c.stream, *a, (int)T, b);
  const size_t ns = (size_t)a->heads * b.Np * (b.Vp / 4);
  const int sb = (int)((ns + 255) / 256), ch = ssm_dims(*a).ch;
  hipLaunchKernelGGL(ssm_scan_kernel, dim3((unsigned)(sb + (ch + 255) / 256)), dim3(256), 0, c.stream, pu, ldu, *a, (int)T, (int)pos0, b, sb);
  auto out = b.C == 64 ? ssm_out_kernel<64> : b.C == 32 ? ssm_out_kernel<32> : ssm_out_kernel<16>;
  e = hipFuncSetAttribute(reinterpret_cast<const void*>(out), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds2);
  if (e != hipSuccess) return hip_fail(e, "hipFuncSetAttribute(LDS)");
  hipLaunchKernelGGL(out, dim3((unsigned)b.np, (unsigned)a->heads), dim3(512), lds2, c.stream, pu, ldu, static_cast<float*>(y), ldy,
                     *a, (int)T, b);
  TLHIP_CHECK_LAUNCH(TLHIP_C_SSM);
}

}  // extern "C"
