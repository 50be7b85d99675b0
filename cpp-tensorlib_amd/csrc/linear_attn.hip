// Prompt chunks of the gated linear attention. The recurrence
//   state row c <- a_c row_c + k_c v,   o = sum_c q_c row_c
// over pieces of C tokens: with b_t the base-2 log of the decay product since the piece began,
//   o_t = (q_t 2^b_t) S_0 + sum_(s <= t) [sum_d q_td k_sd 2^(b_td - b_sd)] v_s
//   S_C = 2^b_C S_0 + sum_s (k_s 2^(b_C - b_s)) v_s^T.
// Three launches: linear_piece_kernel does, for all pieces at once, what needs no state (the second
// term of o, the sum of S_C, the decay products); linear_scan_kernel carries the state through the
// pieces; linear_out_kernel adds the first term and applies norm and gate.
//
// 2^(b_t - b_s) is never formed as 2^b_t 2^-b_s over a whole piece, which overflows under strong
// decays. A piece is cut into blocks of 16 tokens; L_t is the log decay since the block began and tot
// the block's total. Q' = q 2^L_t and K' = k 2^(tot - L_s) have exponents <= 0, and block i sees block
// j < i as  sum_d Q'_td K'_sd 2^(sum of the totals between them). On the diagonal the factor is
// 2^-tot, which is safe while |tot| stays below kFastRange; beyond it the block takes 2^(L_t - L_s)
// pair by pair.
//
// All products run on the fp32 matrix pipe (v_mfma_f32_16x16x4_f32: exact f32 products, fp32 sums).
#include "linear_attn.hpp"

#include <algorithm>

namespace tlhip {

typedef float f32x4 __attribute__((ext_vector_type(4)));
__device__ __forceinline__ f32x4 mfma16(float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

constexpr float kFastRange = 96.f;

// Scratch of a call, per head and piece: decay products [dp], state term [dp][vp]; per head and
// token: decayed query [dp], inner output [vp]. dp, vp: dim and vdim rounded up to 16.
struct PieceBuf {
  float *dec, *st, *qd, *oi;
  int C, np, dp, vp, vs;           // tokens per piece, pieces; vs: value columns of one block of linear_piece_kernel
  int qsh, vsh;                    // its lanes per row of queries and keys, of values: 1 << qsh, 1 << vsh
};

// Four floats of a row of n at column c: zeros past n and where !live. vec: the row starts on 16 bytes
// and n is a multiple of 4.
__device__ __forceinline__ f32x4 load_quad(const float* __restrict__ p, int c, int n, bool vec, bool live) {
  f32x4 x;
  if (vec) {
    x = *reinterpret_cast<const f32x4*>(p + min(c, n - 4));
    if (!live || c >= n) x = f32x4{0.f, 0.f, 0.f, 0.f};
  } else {
#pragma unroll
    for (int j = 0; j < 4; j++) {
      x[j] = p[min(c + j, n - 1)];
      if (!live || c + j >= n) x[j] = 0.f;
    }
  }
  return x;
}
__device__ __forceinline__ f32x4 exp2_quad(f32x4 e) {
  return f32x4{exp2_native(e[0]), exp2_native(e[1]), exp2_native(e[2]), exp2_native(e[3])};
}

// Block (piece of C tokens, head, value slice) of 512 threads. NS: quads of q (and of k) a thread holds.
template <int C, int NS>
__global__ __launch_bounds__(512) void linear_piece_kernel(const float* __restrict__ u, int64_t ldu, const tlhip_linear_attn a,
                                                           int T, const PieceBuf pb) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  constexpr int NB = C / 16, AS = C + 4, NV = (C + 15) / 16;
  const int tid = threadIdx.x, lane = tid & 63, l15 = lane & 15, lg = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int piece = blockIdx.x, h = blockIdx.y, v0 = blockIdx.z * pb.vs;
  const int dp = pb.dp, vp = pb.vp, dim = (int)a.dim, vdim = (int)a.vdim, rank = (int)a.rank;
  const int QS = dp + 4, VS = pb.vs + 4, nv = min(pb.vs, vp - v0), nvl = min(pb.vs, vdim - v0);
  float* Q = lds;                      // [C][QS] Q' (q while a block needs the pairwise form)
  float* K = Q + C * QS;               // [C][QS] K'
  float* Lg = K + C * QS;              // [C][QS] log2 decays since the block began
  float* V = Lg + C * QS;              // [C][VS]
  float* A = V + C * VS;               // [C][AS]
  float* tot = A + C * AS;             // [NB][dp] block totals
  int* slow = reinterpret_cast<int*>(tot + NB * dp);   // [NB]
  const int t0 = piece * C, nt = min(C, T - t0);
  const float inv_tau = 1.0f / a.tau;
  const auto row = [&](int t) { return u + (size_t)(t0 + min(t, nt - 1)) * ldu; };

  // queries, keys and values into registers, 16 bytes a lane: quad i of a thread is token (tid + 512 i) >> sh
  const bool u16 = (reinterpret_cast<uintptr_t>(u) & 15) == 0 && (ldu & 3) == 0;
  const int qo = (int)a.q_off + h * dim, ko = (int)a.k_off + h * dim, vo = (int)a.v_off + h * vdim + v0;
  const bool qvec = u16 && ((qo | ko | dim) & 3) == 0, vvec = u16 && ((vo | nvl) & 3) == 0;
  const int qm = (1 << pb.qsh) - 1, vm = (1 << pb.vsh) - 1;
  f32x4 q[NS], k[NS], v[NV];
#pragma unroll
  for (int i = 0; i < NS; i++) {
    const int slot = tid + 512 * i, t = slot >> pb.qsh, c = 4 * (slot & qm);
    q[i] = load_quad(row(t) + qo, c, dim, qvec, t < nt);
    k[i] = load_quad(row(t) + ko, c, dim, qvec, t < nt);
  }
#pragma unroll
  for (int i = 0; i < NV; i++) {
    const int slot = tid + 512 * i, t = slot >> pb.vsh, c = 4 * (slot & vm);
    v[i] = load_quad(row(t) + vo, c, nvl, vvec, t < nt);
  }
  if (tid < NB) slow[tid] = 0;
  __syncthreads();
  // decay logits Z = low A2^T, a 16 x 16 tile (one block's tokens, 16 channels) at a time; their logs summed
  // up along the tokens: in a lane's four registers, then over the four lane groups
  {
    const uint16_t* a2 = static_cast<const uint16_t*>(a.a2) + (size_t)h * dim * rank;
    const float* bias = static_cast<const float*>(a.bias) + h * dim;
    const bool lvec = u16 && ((rank | (int)a.low_off) & 3) == 0;
    for (int tile = wave; tile < NB * (dp / 16); tile += 8) {
      const int b = tile % NB, d = 16 * (tile / NB) + l15;
      const float* low = row(16 * b + l15) + a.low_off;
      const uint16_t* w = a2 + (size_t)min(d, dim - 1) * rank;
      f32x4 z = {0.f, 0.f, 0.f, 0.f};
      const float bs = bias[min(d, dim - 1)];
      for (int r0 = 0; r0 < rank; r0 += 16) {
        const f32x4 x = load_quad(low, r0 + 4 * lg, rank, lvec, true);
        uint16_t y[4];
#pragma unroll
        for (int j = 0; j < 4; j++) y[j] = w[min(r0 + 4 * lg + j, rank - 1)];   // (x is zero past the rank)
#pragma unroll
        for (int j = 0; j < 4; j++) z = mfma16(x[j], __uint_as_float((uint32_t)y[j] << 16), z);
      }
      float s = 0.f, sum[4];
#pragma unroll
      for (int j = 0; j < 4; j++) {
        const float ld = log2_decay(z[j] + bs, inv_tau);
        s += 16 * b + 4 * lg + j < nt && d < dim ? ld : 0.f;
        sum[j] = s;
      }
      float before = 0.f;                            // of the lane groups below
#pragma unroll
      for (int g = 0; g < 3; g++) {
        const float o = __shfl(s, 16 * g + l15, kWave);
        if (g < lg) before += o;
      }
#pragma unroll
      for (int j = 0; j < 4; j++) Lg[(16 * b + 4 * lg + j) * QS + d] = before + sum[j];
      if (lg == 3) {
        tot[b * dp + d] = before + s;
        if (before + s < -kFastRange) slow[b] = 1;   // (every writer stores the same value)
      }
    }
  }
#pragma unroll
  for (int i = 0; i < NV; i++) {
    const int slot = tid + 512 * i, t = slot >> pb.vsh, c = 4 * (slot & vm);
    if (t < C && c < pb.vs) *reinterpret_cast<f32x4*>(V + t * VS + c) = v[i];
  }
  __syncthreads();
  bool any = false;
#pragma unroll
  for (int b = 0; b < NB; b++) any |= slow[b] != 0;
  if (any) {   // diagonal blocks with strong decays, pair by pair from q and k as they are
#pragma unroll
    for (int i = 0; i < NS; i++) {
      const int slot = tid + 512 * i, t = slot >> pb.qsh, c = 4 * (slot & qm);
      if (t < C && c < dp) {
        *reinterpret_cast<f32x4*>(Q + t * QS + c) = q[i];
        *reinterpret_cast<f32x4*>(K + t * QS + c) = k[i];
      }
    }
    __syncthreads();
    for (int b = 0; b < NB; b++) {
      if (!slow[b] || tid >= 256) continue;
      const int t = 16 * b + tid / 16, s = 16 * b + tid % 16;
      float acc = 0.f;
      if (s <= t)
        for (int d = 0; d < dim; d++) acc = fmaf(Q[t * QS + d] * K[s * QS + d], exp2_native(Lg[t * QS + d] - Lg[s * QS + d]), acc);
      A[t * AS + s] = acc * a.q_scale;
    }
    __syncthreads();
  }
  // Q' and K'; decayed queries for linear_out_kernel, and the piece's decay products
  const size_t hp = (size_t)h * pb.np + piece;
#pragma unroll
  for (int i = 0; i < NS; i++) {
    const int slot = tid + 512 * i, t = slot >> pb.qsh, c = 4 * (slot & qm), b = t >> 4;
    if (t >= C || c >= dp) continue;
    const f32x4 L = *reinterpret_cast<const f32x4*>(Lg + t * QS + c), tt = *reinterpret_cast<const f32x4*>(tot + b * dp + c);
    const f32x4 eq = exp2_quad(L), ek = exp2_quad(tt - L);
    f32x4 x, y, e = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int j = 0; j < 4; j++) { x[j] = q[i][j] * a.q_scale * eq[j]; y[j] = k[i][j] * ek[j]; }
    *reinterpret_cast<f32x4*>(Q + t * QS + c) = x;
    *reinterpret_cast<f32x4*>(K + t * QS + c) = y;
    if (blockIdx.z == 0) {
#pragma unroll
      for (int m = 0; m < NB - 1; m++)
        if (m < b) e += *reinterpret_cast<const f32x4*>(tot + m * dp + c);
      *reinterpret_cast<f32x4*>(pb.qd + (hp * C + t) * dp + c) = x * exp2_quad(e);
    }
  }
  if (blockIdx.z == 0)
    for (int d = tid; d < dp; d += 512) {
      float e = 0.f;
#pragma unroll
      for (int m = 0; m < NB; m++) e += tot[m * dp + d];
      pb.dec[hp * dp + d] = exp2_native(e);
    }
  __syncthreads();
  // A[t][s]: 16 x 16 tiles on and below the diagonal, dealt over the wavefronts
  for (int tile = wave; tile < NB * (NB + 1) / 2; tile += 8) {
    int i = 0, j = tile;
    while (j > i) { i++; j -= i; }
    if (i == j && slow[i]) continue;
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    for (int d0 = 0; d0 < dp; d0 += 16) {
      const int d = d0 + 4 * lg;
      f32x4 qf = *reinterpret_cast<const f32x4*>(Q + (16 * i + l15) * QS + d);
      const f32x4 kf = *reinterpret_cast<const f32x4*>(K + (16 * j + l15) * QS + d);
      if (i == j) {
        qf *= exp2_quad(-*reinterpret_cast<const f32x4*>(tot + i * dp + d));
      } else if (i > j + 1) {
        f32x4 e = {0.f, 0.f, 0.f, 0.f};
        for (int m = j + 1; m < i; m++) e += *reinterpret_cast<const f32x4*>(tot + m * dp + d);
        qf *= exp2_quad(e);
      }
#pragma unroll
      for (int n = 0; n < 4; n++) acc = mfma16(qf[n], kf[n], acc);
    }
#pragma unroll
    for (int n = 0; n < 4; n++) {
      const int t = 4 * lg + n;
      A[(16 * i + t) * AS + 16 * j + l15] = i == j && l15 > t ? 0.f : acc[n];
    }
  }
  // state term: sum over s of K'_sd 2^(totals after s's block) V_sv; four value tiles share the keys
  const int groups = (nv / 16 + 3) / 4;
  for (int tile = wave; tile < (dp / 16) * groups; tile += 8) {
    const int dt = tile / groups, vt = 4 * (tile % groups), d = 16 * dt + l15;
    const int n4 = min(4, nv / 16 - vt);
    f32x4 acc[4];
#pragma unroll
    for (int n = 0; n < 4; n++) acc[n] = f32x4{0.f, 0.f, 0.f, 0.f};
    float e = 0.f;
#pragma unroll
    for (int b = NB - 1; b >= 0; b--) {
      const float w = exp2_native(e);
#pragma unroll
      for (int j = 0; j < 4; j++) {
        const int s = 16 * b + 4 * lg + j;
        const float kw = K[s * QS + d] * w;
#pragma unroll
        for (int n = 0; n < 4; n++) acc[n] = mfma16(kw, V[s * VS + 16 * (vt + min(n, n4 - 1)) + l15], acc[n]);
      }
      e += tot[b * dp + d];
    }
#pragma unroll
    for (int n = 0; n < 4; n++)
      if (n < n4)
#pragma unroll
        for (int j = 0; j < 4; j++) pb.st[(hp * dp + 16 * dt + 4 * lg + j) * vp + v0 + 16 * (vt + n) + l15] = acc[n][j];
  }
  __syncthreads();
  // inner output: A V; the two wavefronts of a SIMD take a long and a short row of blocks
  for (int tile = wave; tile < NB * groups; tile += 8) {
    const int f = tile % NB, i = (tile / NB) & 1 ? NB - 1 - f : f, vt = 4 * (tile / NB), n4 = min(4, nv / 16 - vt);
    f32x4 acc[4];
#pragma unroll
    for (int n = 0; n < 4; n++) acc[n] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int b = 0; b <= i; b++) {
      const int s = 16 * b + 4 * lg;
      const f32x4 p = *reinterpret_cast<const f32x4*>(A + (16 * i + l15) * AS + s);
#pragma unroll
      for (int j = 0; j < 4; j++)
#pragma unroll
        for (int n = 0; n < 4; n++) acc[n] = mfma16(p[j], V[(s + j) * VS + 16 * (vt + min(n, n4 - 1)) + l15], acc[n]);
    }
#pragma unroll
    for (int n = 0; n < 4; n++)
      if (n < n4)
#pragma unroll
        for (int j = 0; j < 4; j++) pb.oi[(hp * C + 16 * i + 4 * lg + j) * vp + v0 + 16 * (vt + n) + l15] = acc[n][j];
  }
}

// The state through the pieces: st[piece] becomes the state ahead of the piece, the last state goes to
// its slot. A thread owns four value columns of one row.
__global__ __launch_bounds__(256) void linear_scan_kernel(const tlhip_linear_attn a, int T, int pos0, const PieceBuf pb) {
  const int dim = (int)a.dim, ld = (int)linear_state_ld(a.vdim), nv4 = pb.vp / 4;
  const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= (size_t)a.heads * pb.dp * nv4) return;
  const int v = 4 * (int)(i % nv4), d = (int)(i / nv4 % pb.dp), h = (int)(i / nv4 / pb.dp);
  const size_t slot = (size_t)a.heads * dim * ld, at = ((size_t)h * dim + d) * ld + v;
  const bool kept = d < dim && v < ld;
  float* state = static_cast<float*>(a.state);
  float4 s = make_float4(0.f, 0.f, 0.f, 0.f);
  if (kept && pos0 > 0) s = *reinterpret_cast<const float4*>(state + (size_t)(pos0 & 1) * slot + at);
  constexpr int U = 8;                               // pieces requested at once
  for (int p0 = 0; p0 < pb.np; p0 += U) {
    float4 t[U];
    float w[U];
#pragma unroll
    for (int k = 0; k < U; k++) {
      const size_t hp = (size_t)h * pb.np + min(p0 + k, pb.np - 1);
      t[k] = *reinterpret_cast<const float4*>(pb.st + (hp * pb.dp + d) * pb.vp + v);
      w[k] = pb.dec[hp * pb.dp + d];
    }
#pragma unroll
    for (int k = 0; k < U; k++)
      if (p0 + k < pb.np) {
        const size_t hp = (size_t)h * pb.np + p0 + k;
        *reinterpret_cast<float4*>(pb.st + (hp * pb.dp + d) * pb.vp + v) = s;
        s.x = fmaf(w[k], s.x, t[k].x); s.y = fmaf(w[k], s.y, t[k].y); s.z = fmaf(w[k], s.z, t[k].z); s.w = fmaf(w[k], s.w, t[k].w);
      }
  }
  if (kept) *reinterpret_cast<float4*>(state + (size_t)((pos0 + T) & 1) * slot + at) = s;
}

// Block (TM tokens, head) of 512 threads: the state's part of o, norm over vdim, gate.
template <int MT>
__global__ __launch_bounds__(512) void linear_out_kernel(const float* __restrict__ u, int64_t ldu, float* __restrict__ y,
                                                         int64_t ldy, const tlhip_linear_attn a, int T, const PieceBuf pb) {
  constexpr int TM = 16 * MT;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int tid = threadIdx.x, lane = tid & 63, l15 = lane & 15, lg = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int t0 = blockIdx.x * TM, h = blockIdx.y, dp = pb.dp, vp = pb.vp, OS = vp + 4, vdim = (int)a.vdim;
  const size_t hp = (size_t)h * pb.np + t0 / pb.C, hr = (size_t)h * pb.np * pb.C + t0;
  // what the end of the kernel needs of u, requested now: norm weights and gates of the first 128 columns
  float gate[TM / 8][2], nrm[2];
#pragma unroll
  for (int c = 0; c < 2; c++) {
    const int v = min(lane + 64 * c, vdim - 1);
    nrm[c] = static_cast<const float*>(a.norm)[v];
#pragma unroll
    for (int i = 0; i < TM / 8; i++) gate[i][c] = u[(size_t)min(t0 + wave + 8 * i, T - 1) * ldu + a.gate_off + (int64_t)h * vdim + v];
  }
  for (int vt = wave; vt < vp / 16; vt += 8) {
    f32x4 acc[MT];
#pragma unroll
    for (int mt = 0; mt < MT; mt++)
#pragma unroll
      for (int v = 0; v < 4; v++) acc[mt][v] = pb.oi[(hr + 16 * mt + 4 * lg + v) * vp + 16 * vt + l15];
    for (int d1 = 0; d1 < dp; d1 += 64) {            // four steps requested at once (past dp: clamped, times zero)
      float sv[4][4];
      f32x4 q[4][MT];
#pragma unroll
      for (int k = 0; k < 4; k++) {
        const int d = min(d1 + 16 * k, dp - 16) + 4 * lg;
        const float* sp = pb.st + (hp * dp + d) * vp + 16 * vt + l15;
#pragma unroll
        for (int j = 0; j < 4; j++) sv[k][j] = sp[j * vp];
#pragma unroll
        for (int mt = 0; mt < MT; mt++) q[k][mt] = *reinterpret_cast<const f32x4*>(pb.qd + (hr + 16 * mt + l15) * dp + d);
      }
#pragma unroll
      for (int k = 0; k < 4; k++)
#pragma unroll
        for (int mt = 0; mt < MT; mt++)
#pragma unroll
          for (int j = 0; j < 4; j++) acc[mt] = mfma16(d1 + 16 * k < dp ? q[k][mt][j] : 0.f, sv[k][j], acc[mt]);
    }
#pragma unroll
    for (int mt = 0; mt < MT; mt++)
#pragma unroll
      for (int v = 0; v < 4; v++) lds[(16 * mt + 4 * lg + v) * OS + 16 * vt + l15] = acc[mt][v];
  }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < TM / 8; i++) {
    const int r = wave + 8 * i;
    if (t0 + r >= T) break;
    float ss = 0.f;
    for (int v = lane; v < vdim; v += 64) ss = fmaf(lds[r * OS + v], lds[r * OS + v], ss);
    ss = wave_sum(ss);
    const float inv = 1.0f / sqrtf(ss / (float)vdim + a.eps);
    float* o = y + (size_t)(t0 + r) * ldy + a.y_off + (int64_t)h * vdim;
#pragma unroll
    for (int c = 0; c < 2; c++) {
      const int v = lane + 64 * c;
      if (v < vdim) o[v] = lds[r * OS + v] * inv * nrm[c] * (gate[i][c] * sigmoid_f(gate[i][c])) * a.out_scale;
    }
    const float* g = u + (size_t)(t0 + r) * ldu + a.gate_off + (int64_t)h * vdim;
    for (int v = lane + 128; v < vdim; v += 64)
      o[v] = lds[r * OS + v] * inv * static_cast<const float*>(a.norm)[v] * (g[v] * sigmoid_f(g[v])) * a.out_scale;
  }
}

static size_t piece_lds(int C, int dp, int vs) {
  return (size_t)(3 * C * (dp + 4) + C * (vs + 4) + C * (C + 4) + (C / 16) * dp + 16) * sizeof(float);
}

}  // namespace tlhip

using namespace tlhip;

extern "C" {

int tlhip_linear_attn_chunk(const void* u, int64_t ldu, void* y, int64_t ldy, const tlhip_linear_attn* la, int64_t T,
                            int64_t pos0) {
  TLHIP_REQUIRE_READY();
  if (!u || !y || !la || ldu <= 0 || ldy <= 0) return fail(TLHIP_EINVAL, "tlhip_linear_attn_chunk: bad operands");
  if (T <= 0 || T > (1 << 20) || pos0 < 0 || pos0 + T > (1 << 30)) return fail(TLHIP_EINVAL, "tlhip_linear_attn_chunk: bad chunk");
  if (int rc = check_linear_attn(la, "tlhip_linear_attn_chunk")) return rc;
  Context& c = ctx();
  PieceBuf pb{};
  pb.dp = (int)(la->dim + 15) / 16 * 16;
  pb.vp = (int)(la->vdim + 15) / 16 * 16;
  pb.C = 64;
  while (pb.C > 16 && (piece_lds(pb.C, pb.dp, 64) > (size_t)c.lds_per_cu || pb.C / 2 >= T)) pb.C /= 2;
  pb.vs = std::min(pb.vp, 128);        // every slice of values repeats the work on queries and keys
  if (piece_lds(pb.C, pb.dp, pb.vs) > (size_t)c.lds_per_cu) pb.vs = 64;
  const size_t lds1 = piece_lds(pb.C, pb.dp, pb.vs);
  const int mt = pb.C >= 32 ? 2 : 1;
  const size_t lds3 = (size_t)16 * mt * (pb.vp + 4) * sizeof(float);
  if (lds1 > (size_t)c.lds_per_cu || lds3 > (size_t)c.lds_per_cu)
    return fail(TLHIP_EUNSUPPORTED, "tlhip_linear_attn_chunk: head too large for LDS");
  pb.np = (int)((T + pb.C - 1) / pb.C);
  const size_t hp = (size_t)la->heads * pb.np, n_dec = hp * pb.dp, n_st = hp * pb.dp * pb.vp, n_qd = hp * pb.C * pb.dp,
               n_oi = hp * pb.C * pb.vp;
  float* s = static_cast<float*>(scratch((n_dec + n_st + n_qd + n_oi) * sizeof(float)));
  if (!s) return fail(TLHIP_ENOMEM, "tlhip_linear_attn_chunk: no scratch");
  pb.dec = s;
  pb.st = pb.dec + n_dec;
  pb.qd = pb.st + n_st;
  pb.oi = pb.qd + n_qd;
  const float* pu = static_cast<const float*>(u);
  while (4 << pb.qsh < pb.dp) pb.qsh++;
  while (4 << pb.vsh < pb.vs) pb.vsh++;
  const int quads = ((pb.C << pb.qsh) + 511) / 512;   // of queries (and keys) per thread
  void (*piece)(const float*, int64_t, tlhip_linear_attn, int, PieceBuf) = nullptr;
#define TLHIP_PIECE(C) (quads <= 2 ? linear_piece_kernel<C, 2> : quads <= 4 ? linear_piece_kernel<C, 4> : quads <= 8 ? linear_piece_kernel<C, 8> : nullptr)
  piece = pb.C == 64 ? TLHIP_PIECE(64) : pb.C == 32 ? TLHIP_PIECE(32) : TLHIP_PIECE(16);
#undef TLHIP_PIECE
  if (!piece) return fail(TLHIP_EUNSUPPORTED, "tlhip_linear_attn_chunk: no kernel for this head size");
  hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(piece), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds1);
  if (e != hipSuccess) return hip_fail(e, "hipFuncSetAttribute(LDS)");
  hipLaunchKernelGGL(piece, dim3((unsigned)pb.np, (unsigned)la->heads, (unsigned)((pb.vp + pb.vs - 1) / pb.vs)), dim3(512), lds1,
                     c.stream, pu, ldu, *la, (int)T, pb);
  const size_t ns = (size_t)la->heads * pb.dp * (pb.vp / 4);
  hipLaunchKernelGGL(linear_scan_kernel, dim3((unsigned)((ns + 255) / 256)), dim3(256), 0, c.stream, *la, (int)T, (int)pos0, pb);
  auto out = mt == 2 ? linear_out_kernel<2> : linear_out_kernel<1>;
  e = hipFuncSetAttribute(reinterpret_cast<const void*>(out), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds3);
  if (e != hipSuccess) return hip_fail(e, "hipFuncSetAttribute(LDS)");
  hipLaunchKernelGGL(out, dim3((unsigned)((T + 16 * mt - 1) / (16 * mt)), (unsigned)la->heads), dim3(512), lds3, c.stream, pu, ldu,
                     static_cast<float*>(y), ldy, *la, (int)T, pb);
  TLHIP_CHECK_LAUNCH(TLHIP_C_LINEAR_ATTN);
}

}  // extern "C"
