// Row ops around the layers: token rows with sinusoidal positions, sums into the residual stream, row
// gathers, the PolyNorm activation of a chunk.
#include "common.hpp"
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

}  // extern "C"
