// Row ops around the layers: token rows with sinusoidal positions, sums into the residual stream, row
// gathers, norms of what a sublayer wrote, the PolyNorm and gated GELU activations of a chunk.
#include "common.hpp"
#include "gemv_shared.hpp"
#include "polynorm.hpp"

namespace tlhip {

// Angles in double: a position times a frequency loses digits in fp32 at positions in the thousands.
__global__ __launch_bounds__(256) void embed_sinusoid_kernel(const uint16_t* __restrict__ table, const int* __restrict__ tokens,
                                                             float* __restrict__ out, int width, int ld, int vocab, int pos0,
                                                             const uint32_t* __restrict__ d_pos) {
  const int c = blockIdx.x * 256 + threadIdx.x, t = blockIdx.y;
  if (c >= ld) return;
  const int p = (d_pos ? (int)*d_pos : pos0) + t;
  int tok = tokens[t];
  tok = tok < 0 ? 0 : (tok >= vocab ? vocab - 1 : tok);
  float v = 0.f;
  if (c < width) {
    const double ang = (double)p * exp(-(double)(c & ~1) / (double)width * 9.210340371976184);   // ln 10000
    v = __uint_as_float((uint32_t)table[(size_t)tok * width + c] << 16) + (float)((c & 1) ? cos(ang) : sin(ang));
  }
  out[(size_t)t * ld + c] = v;
}

__global__ __launch_bounds__(256) void residual_sum_kernel(const float* x, const float* __restrict__ parts, int S,
                                                           const float* __restrict__ add, const float* __restrict__ vec,
                                                           float* out, int n, size_t total) {
  const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= total) return;
  float v = x[i];
  for (int s = 0; s < S; s++) v += parts[s * total + i];
  if (add) v += add[i];
  if (vec) v += vec[i % n];
  out[i] = v;
}

__global__ __launch_bounds__(256) void gather_rows_kernel(const float* __restrict__ src, const int* __restrict__ idx,
                                                          float* __restrict__ out, int n, int src_rows) {
  const int r = min(max(idx[blockIdx.y], 0), src_rows - 1), c = blockIdx.x * 256 + threadIdx.x;
  if (c < n) out[(size_t)blockIdx.y * n + c] = src[(size_t)r * n + c];
}

// L > 0: rows held in registers (polynorm_row), else any row
template <int L>
__global__ __launch_bounds__(512) void polynorm_rows_kernel(const float* __restrict__ u, int64_t ldu, float* __restrict__ y,
                                                            int64_t ldy, const tlhip_polynorm p) {
  __shared__ float red[24];
  const float* z = u + (size_t)blockIdx.x * ldu + p.z_off;
  float* o = y + (size_t)blockIdx.x * ldy + p.y_off;
  if constexpr (L > 0) polynorm_row<512, L>(p, z, o, red);
  else polynorm_block<512>(p, z, o, 0, (int)p.ff, red);
}

__global__ __launch_bounds__(256) void embed_scaled_kernel(const uint16_t* __restrict__ table, int64_t ldt,
                                                           const int* __restrict__ tokens, float* __restrict__ out, int width,
                                                           int ld, int vocab, float scale) {
  const int c = blockIdx.x * 256 + threadIdx.x, t = blockIdx.y;
  if (c >= ld) return;
  const int tok = min(max(tokens[t], 0), vocab - 1);
  out[(size_t)t * ld + c] = c < width ? __uint_as_float((uint32_t)table[(size_t)tok * ldt + c] << 16) * scale : 0.f;
}

// xout = x + rms(parts + bias) * w, one block of 1024 threads per row, RV float4s a thread.
template <int RV>
__global__ __launch_bounds__(1024) void postnorm_rows_kernel(const float* x, const float* __restrict__ delta, int S,
                                                             size_t part_stride, const float* __restrict__ bias,
                                                             const float* __restrict__ w, float* xout, int n, float eps) {
  __shared__ float red[16];
  const size_t base = (size_t)blockIdx.x * n;
  const int n4 = n >> 2;
  float4 v[RV], xv[RV], wv[RV];
  float acc = 0.f;
#pragma unroll
  for (int k = 0; k < RV; k++) {
    const int i = threadIdx.x + k * 1024;
    if (i < n4) {
      const float4* d4 = reinterpret_cast<const float4*>(delta + base);
      xv[k] = reinterpret_cast<const float4*>(x + base)[i];
      wv[k] = reinterpret_cast<const float4*>(w)[i];
      v[k] = d4[i];
      for (int s = 1; s < S; s++) {    // K-split parts, ascending
        const float4 e = d4[s * (part_stride >> 2) + i];
        v[k].x += e.x; v[k].y += e.y; v[k].z += e.z; v[k].w += e.w;
      }
      if (bias) {
        const float4 e = reinterpret_cast<const float4*>(bias)[i];
        v[k].x += e.x; v[k].y += e.y; v[k].z += e.z; v[k].w += e.w;
      }
      acc += (v[k].x * v[k].x + v[k].y * v[k].y) + (v[k].z * v[k].z + v[k].w * v[k].w);
    }
  }
  const float inv = 1.0f / sqrtf(block_sum<16>(acc, red) / (float)n + eps);
#pragma unroll
  for (int k = 0; k < RV; k++) {
    const int i = threadIdx.x + k * 1024;
    if (i < n4)
      reinterpret_cast<float4*>(xout + base)[i] =
          make_float4(fmaf(v[k].x * inv, wv[k].x, xv[k].x), fmaf(v[k].y * inv, wv[k].y, xv[k].y),
                      fmaf(v[k].z * inv, wv[k].z, xv[k].z), fmaf(v[k].w * inv, wv[k].w, xv[k].w));
  }
}

// Block (row) of 256 threads; a wavefront norms whole runs, or the four share one where there are fewer than four.
// VEC: runs and rows of whole float4s. A thread keeps up to kKeep of its entries.
template <bool VEC>
__global__ __launch_bounds__(256) void rms_rows_kernel(const float* x, int64_t ldx, const float* __restrict__ w, float* out,
                                                       int64_t ldo, int n, int n_out, int parts, float eps) {
  typedef float vec __attribute__((ext_vector_type(VEC ? 4 : 1)));
  constexpr int E = VEC ? 4 : 1, kKeep = 4;
  __shared__ float red[4];
  const int tid = threadIdx.x, len = n / parts / E;
  const bool whole = parts < 4;        // the block shares a run
  const int at = whole ? tid : tid & 63, step = whole ? 256 : 64;
  float* o = out + (size_t)blockIdx.x * ldo;
  for (int p = whole ? 0 : tid >> 6; p < parts; p += whole ? 1 : 4) {
    const vec* r = reinterpret_cast<const vec*>(x + (size_t)blockIdx.x * ldx) + p * len;
    const vec* wr = reinterpret_cast<const vec*>(w) + p * len;
    vec* q = reinterpret_cast<vec*>(o) + p * len;
    const auto square = [](vec v) {
      float s = 0.f;
#pragma unroll
      for (int e = 0; e < E; e++) s = fmaf(v[e], v[e], s);
      return s;
    };
    vec v[kKeep];
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < kKeep; k++) v[k] = r[min(at + k * step, len - 1)];
#pragma unroll
    for (int k = 0; k < kKeep; k++)
      if (at + k * step < len) ss += square(v[k]);
    for (int i = at + kKeep * step; i < len; i += step) ss += square(r[i]);
    const float inv = 1.0f / sqrtf((whole ? block_sum<4>(ss, red) : wave_sum(ss)) / (float)(len * E) + eps);
#pragma unroll
    for (int k = 0; k < kKeep; k++)
      if (at + k * step < len) q[at + k * step] = v[k] * inv * wr[at + k * step];
    for (int i = at + kKeep * step; i < len; i += step) q[i] = r[i] * inv * wr[i];
  }
  for (int i = n + tid; i < n_out; i += 256) o[i] = 0.f;
}

__global__ __launch_bounds__(256) void geglu_rows_kernel(const float* __restrict__ gu, const float* __restrict__ bias,
                                                         float* __restrict__ out, int ff) {
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i >= ff) return;
  const float* r = gu + (size_t)blockIdx.y * 2 * ff;
  out[(size_t)blockIdx.y * ff + i] = gelu_tanh(r[i] + bias[i]) * (r[ff + i] + bias[ff + i]);
}

}  // namespace tlhip

using namespace tlhip;

extern "C" {

int tlhip_embed_sinusoid(const void* table, const void* tokens, void* out, int64_t T, int64_t width, int64_t ld, int64_t vocab,
                         int64_t pos0, const void* d_pos) {
  TLHIP_REQUIRE_READY();
  if (!table || !tokens || !out) return fail(TLHIP_EINVAL, "tlhip_embed_sinusoid: null pointer");
  if (T <= 0 || T > 65535 || width <= 0 || ld < width || vocab <= 0 || pos0 < 0 || pos0 + T > (1 << 30))
    return fail(TLHIP_EINVAL, "tlhip_embed_sinusoid: bad sizes");
  embed_sinusoid_kernel<<<dim3((unsigned)((ld + 255) / 256), (unsigned)T), dim3(256), 0, ctx().stream>>>(
      static_cast<const uint16_t*>(table), static_cast<const int*>(tokens), static_cast<float*>(out), (int)width, (int)ld,
      (int)vocab, (int)pos0, static_cast<const uint32_t*>(d_pos));
  TLHIP_CHECK_LAUNCH(TLHIP_C_EMBED);
}

int tlhip_residual_sum(const void* x, const void* parts, int64_t S, const void* add, const void* vec, void* out, int64_t n,
                       int64_t rows) {
  TLHIP_REQUIRE_READY();
  if (!x || !out || n <= 0 || rows <= 0 || S < 0 || S > 64 || n > (1 << 30)) return fail(TLHIP_EINVAL, "tlhip_residual_sum: bad operands");
  const size_t total = (size_t)n * rows;
  residual_sum_kernel<<<dim3((unsigned)((total + 255) / 256)), dim3(256), 0, ctx().stream>>>(
      static_cast<const float*>(x), static_cast<const float*>(parts), parts ? (int)S : 0, static_cast<const float*>(add),
      static_cast<const float*>(vec), static_cast<float*>(out), (int)n, total);
  TLHIP_CHECK_LAUNCH(TLHIP_C_RESIDUAL);
}

int tlhip_gather_rows(const void* src, const void* idx, void* out, int64_t n, int64_t rows, int64_t src_rows) {
  TLHIP_REQUIRE_READY();
  if (!src || !idx || !out || n <= 0 || rows <= 0 || rows > 65535 || src_rows <= 0 || n > (1 << 30) || src_rows > (1 << 30))
    return fail(TLHIP_EINVAL, "tlhip_gather_rows: bad operands");
  gather_rows_kernel<<<dim3((unsigned)((n + 255) / 256), (unsigned)rows), dim3(256), 0, ctx().stream>>>(
      static_cast<const float*>(src), static_cast<const int*>(idx), static_cast<float*>(out), (int)n, (int)src_rows);
  TLHIP_CHECK_LAUNCH(TLHIP_C_EMBED);
}

int tlhip_polynorm_rows(const void* u, int64_t ldu, void* y, int64_t ldy, const tlhip_polynorm* pn, int64_t T) {
  TLHIP_REQUIRE_READY();
  if (!u || !y || !pn || !aligned16(u) || ldu <= 0 || ldu % 4 || ldy <= 0 || T <= 0 || T > (1 << 30))
    return fail(TLHIP_EINVAL, "tlhip_polynorm_rows: bad operands");
  if (int rc = check_polynorm(pn, "tlhip_polynorm_rows")) return rc;
  const bool vec = pn->ff % 4 == 0 && ldy % 4 == 0 && pn->y_off % 4 == 0 && aligned16(y);
  const int64_t per = (pn->ff / 4 + 511) / 512;
  auto fn = !vec || per > 12 ? polynorm_rows_kernel<0> : per <= 3 ? polynorm_rows_kernel<3> : per <= 6 ? polynorm_rows_kernel<6>
                                                       : polynorm_rows_kernel<12>;
  hipLaunchKernelGGL(fn, dim3((unsigned)T), dim3(512), 0, ctx().stream, static_cast<const float*>(u), ldu, static_cast<float*>(y), ldy,
                     *pn);
  TLHIP_CHECK_LAUNCH(TLHIP_C_POLYNORM);
}

int tlhip_embed_scaled(const void* table, int64_t ldt, const void* tokens, void* out, int64_t T, int64_t width, int64_t ld,
                       int64_t vocab, float scale) {
  TLHIP_REQUIRE_READY();
  if (!table || !tokens || !out) return fail(TLHIP_EINVAL, "tlhip_embed_scaled: null pointer");
  if (T <= 0 || T > 65535 || width <= 0 || ldt < width || ld < width || vocab <= 0 || ld > (1 << 30) || vocab > (1 << 30))
    return fail(TLHIP_EINVAL, "tlhip_embed_scaled: bad sizes");
  embed_scaled_kernel<<<dim3((unsigned)((ld + 255) / 256), (unsigned)T), dim3(256), 0, ctx().stream>>>(
      static_cast<const uint16_t*>(table), ldt, static_cast<const int*>(tokens), static_cast<float*>(out), (int)width, (int)ld,
      (int)vocab, scale);
  TLHIP_CHECK_LAUNCH(TLHIP_C_EMBED);
}

int tlhip_postnorm_res_parts(const void* x, const void* parts, int64_t S, const void* bias, const void* norm_w, void* xout,
                             int64_t n, float eps, int64_t rows, void* aimage) {
  TLHIP_REQUIRE_READY();
  const char* who = "tlhip_postnorm_res_parts";
  if (!x || !parts || !norm_w || !xout) return fail(TLHIP_EINVAL, "%s: null pointer", who);
  if (n <= 0 || n % 4 || n > 32768 || rows <= 0 || rows > (1 << 24) || S < 1 || S > 64)
    return fail(TLHIP_EUNSUPPORTED, "%s: need n %% 4 == 0, n <= 32768, rows and 1 <= S <= 64", who);
  if (!aligned16(x) || !aligned16(parts) || !aligned16(norm_w) || !aligned16(xout) || (bias && !aligned16(bias)))
    return fail(TLHIP_EINVAL, "%s: misaligned", who);
  if (xout == parts) return fail(TLHIP_EINVAL, "%s: xout must not alias the parts", who);
  if (aimage)
    return postnorm_aimage(static_cast<const float*>(x), static_cast<const float*>(parts), (int)S, static_cast<const float*>(bias),
                           static_cast<const float*>(norm_w), static_cast<float*>(xout), (int)n, eps, (int)rows, aimage);
  auto fn = n <= 4096 ? postnorm_rows_kernel<1> : n <= 8192 ? postnorm_rows_kernel<2> : postnorm_rows_kernel<8>;
  hipLaunchKernelGGL(fn, dim3((unsigned)rows), dim3(1024), 0, ctx().stream, static_cast<const float*>(x), static_cast<const float*>(parts),
                     (int)S, (size_t)(rows * n), static_cast<const float*>(bias), static_cast<const float*>(norm_w),
                     static_cast<float*>(xout), (int)n, eps);
  TLHIP_CHECK_LAUNCH(TLHIP_C_RMSNORM_RES);
}

int tlhip_rms_rows(const void* x, int64_t ldx, const void* w, void* out, int64_t ldo, int64_t n, int64_t n_out, int64_t parts,
                   float eps, int64_t rows) {
  TLHIP_REQUIRE_READY();
  if (!x || !w || !out) return fail(TLHIP_EINVAL, "tlhip_rms_rows: null pointer");
  if (n <= 0 || n_out < n || n_out > (1 << 30) || ldx < n || ldo < n_out || parts <= 0 || n % parts || rows <= 0 || rows > (1 << 30))
    return fail(TLHIP_EINVAL, "tlhip_rms_rows: bad sizes");
  const bool vec = n / parts % 4 == 0 && ldx % 4 == 0 && ldo % 4 == 0 && aligned16(x) && aligned16(w) && aligned16(out);
  hipLaunchKernelGGL(vec ? rms_rows_kernel<true> : rms_rows_kernel<false>, dim3((unsigned)rows), dim3(256), 0, ctx().stream,
                     static_cast<const float*>(x), ldx, static_cast<const float*>(w), static_cast<float*>(out), ldo, (int)n, (int)n_out,
                     (int)parts, eps);
  TLHIP_CHECK_LAUNCH(TLHIP_C_RMSNORM);
}

int tlhip_geglu_rows(const void* gu, const void* bias, void* out, int64_t ff, int64_t rows) {
  TLHIP_REQUIRE_READY();
  if (!gu || !bias || !out || ff <= 0 || ff > (1 << 29) || rows <= 0 || rows > 65535) return fail(TLHIP_EINVAL, "tlhip_geglu_rows: bad operands");
  geglu_rows_kernel<<<dim3((unsigned)((ff + 255) / 256), (unsigned)rows), dim3(256), 0, ctx().stream>>>(
      static_cast<const float*>(gu), static_cast<const float*>(bias), static_cast<float*>(out), (int)ff);
  TLHIP_CHECK_LAUNCH(TLHIP_C_ACT);
}

}  // extern "C"
