// The decode step of a layer whose sublayers stand side by side: one launch over the row u that the
// layer's one projection wrote, different blocks doing different sublayers
//   [attention: kv head x query-head subgroup x split | linear attention: head | polynorm: slice of ff]
// each writing its columns of y, the input of the layer's one output product. Where the window is
// cut into splits a second launch merges them.
#include "attn_window.hpp"
#include "linear_attn.hpp"
#include "polynorm.hpp"

#include <algorithm>

namespace tlhip {

struct MixPlan {
  int nq;            // query heads per attention block
  int subs;          // query-head subgroups per kv head
  int S;             // splits of the window
  int attn, lin, poly;   // blocks of each kind
};
constexpr int kPolySlice = 1024;   // ff values a polynorm block writes
constexpr int kMaxSplits = 32;

static int attn_splits(const tlhip_window_attn* a) {
  // What a block reads bounds it (a CU takes in some 100 bytes per ns): windows beyond 192 KB of keys are
  // cut into splits of about 64 KB, which costs the merge launch. The plan does not depend on the position.
  const int64_t bytes = a->window * tlhip_window_ring_ld(a->dim) * 4, S = bytes <= (192 << 10) ? 1 : (bytes + (64 << 10) - 1) / (64 << 10);
  return (int)(S > kMaxSplits ? kMaxSplits : S);
}
static MixPlan make_plan(const tlhip_window_attn* at, const tlhip_linear_attn* la, const tlhip_polynorm* pn) {
  MixPlan p{1, 0, 1, 0, 0, 0};
  if (at) {
    const int group = (int)(at->heads / at->kv_heads), cus = ctx().cus > 0 ? ctx().cus : 256;
    p.S = attn_splits(at);
    // one query head per block while that fits the chip in one round; more share a block's key reads
    const auto blocks = [&](int nq) { return at->kv_heads * ((group + nq - 1) / nq) * p.S; };
    const int most = at->ring_ld > 128 ? 2 : 4;   // registers
    p.nq = 1;
    while (p.nq < most && p.nq < group && blocks(p.nq) > cus) p.nq *= 2;
    p.subs = (group + p.nq - 1) / p.nq;
    p.attn = (int)blocks(p.nq);
  }
  if (la) p.lin = (int)la->heads;
  if (pn) p.poly = (int)((pn->ff + kPolySlice - 1) / kPolySlice);
  return p;
}

template <int NQ, int NF>
__global__ __launch_bounds__(512) void mix_step_kernel(const float* __restrict__ u, float* __restrict__ y,
                                                       const tlhip_window_attn at, const tlhip_linear_attn la,
                                                       const tlhip_polynorm pn, float* __restrict__ partials, int pos,
                                                       const uint32_t* __restrict__ d_pos, const MixPlan plan) {
  extern __shared__ __attribute__((aligned(16))) float mix_lds[];
  int b = blockIdx.x;
  const int p = d_pos ? (int)*d_pos : pos;
  if (b < plan.attn) {
    const int split = b % plan.S, r = b / plan.S, sub = r % plan.subs, kvh = r / plan.subs;
    const int group = (int)(at.heads / at.kv_heads), h0 = sub * NQ;
    window_step_block<NQ, NF>(at, u, y, partials, p, kvh, h0, min(NQ, group - h0), split, plan.S, mix_lds);
    return;
  }
  b -= plan.attn;
  if (b < plan.lin) {
    linear_step_block(la, u, y, p, b, mix_lds);
    return;
  }
  b -= plan.lin;
  const int i0 = b * kPolySlice;
  polynorm_block<512>(pn, u + pn.z_off, y + pn.y_off, i0, min(i0 + kPolySlice, (int)pn.ff), mix_lds);
}

__global__ __launch_bounds__(256) void mix_merge_kernel(const float* __restrict__ u, float* __restrict__ y,
                                                        const tlhip_window_attn at, const float* __restrict__ partials,
                                                        int S) {
  window_merge_head(at, u, y, partials, blockIdx.x, S);
}

int check_window_attn(const tlhip_window_attn* a, const char* who) {
  if (a->heads <= 0 || a->kv_heads <= 0 || a->heads % a->kv_heads || a->dim <= 0 || a->window <= 0)
    return fail(TLHIP_EINVAL, "%s: bad attention sizes", who);
  if (!a->ring || !aligned16(a->ring)) return fail(TLHIP_EINVAL, "%s: key ring null or not 16-byte aligned", who);
  if (a->heads > 65535 || a->window > (1 << 30) || a->ring_rows > (1 << 30))
    return fail(TLHIP_EUNSUPPORTED, "%s: attention dimension too large", who);
  if (tlhip_window_ring_ld(a->dim) == 0) return fail(TLHIP_EUNSUPPORTED, "%s: head size beyond 256", who);
  if (a->ring_ld != tlhip_window_ring_ld(a->dim) || a->ring_rows <= 0 || a->ring_rows % 32)
    return fail(TLHIP_EINVAL, "%s: key ring of the wrong shape", who);
  return TLHIP_OK;
}
int check_linear_attn(const tlhip_linear_attn* a, const char* who) {
  if (a->heads <= 0 || a->dim <= 0 || a->vdim <= 0 || a->rank <= 0 || !(a->tau > 0.f))
    return fail(TLHIP_EINVAL, "%s: bad linear attention sizes", who);
  if (!a->a2 || !a->bias || !a->norm || !a->state || !aligned16(a->state))
    return fail(TLHIP_EINVAL, "%s: null or misaligned linear attention operand", who);
  if (a->dim > 512 || a->vdim > 1024 || a->heads > 65535)
    return fail(TLHIP_EUNSUPPORTED, "%s: linear attention heads beyond 512 x 1024", who);
  return TLHIP_OK;
}
int check_polynorm(const tlhip_polynorm* p, const char* who) {
  if (p->ff <= 0 || p->ff > (1 << 30)) return fail(TLHIP_EINVAL, "%s: bad feed-forward size", who);
  if (p->z_off % 4) return fail(TLHIP_EINVAL, "%s: z must start on a 16-byte boundary", who);
  return TLHIP_OK;
}

template <int NQ, int NF>
static int launch_mix(const float* u, float* y, const tlhip_window_attn* at, const tlhip_linear_attn* la,
                      const tlhip_polynorm* pn, int pos, const void* d_pos, float* partials, const MixPlan& plan) {
  Context& c = ctx();
  const tlhip_window_attn a0{};
  const tlhip_linear_attn l0{};
  const tlhip_polynorm p0{};
  size_t lds = 3 * 8 * sizeof(float);
  if (at) lds = std::max(lds, (size_t)8 * NQ * (64 * NF + 2) * sizeof(float));
  if (at) lds = std::max(lds, (size_t)(NQ + 1) * 64 * NF * sizeof(float));
  if (la) lds = std::max(lds, linear_step_lds(la->dim, la->vdim));
  auto fn = mix_step_kernel<NQ, NF>;
  if (lds > (size_t)c.lds_per_cu) return fail(TLHIP_EUNSUPPORTED, "tlhip_mix_step: not enough LDS");
  if (lds > 48 * 1024) {
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(fn), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return hip_fail(e, "hipFuncSetAttribute(LDS)");
  }
  hipLaunchKernelGGL(fn, dim3((unsigned)(plan.attn + plan.lin + plan.poly)), dim3(512), lds, c.stream, u, y,
                     at ? *at : a0, la ? *la : l0, pn ? *pn : p0, partials, pos, static_cast<const uint32_t*>(d_pos), plan);
  if (at && plan.S > 1)
    hipLaunchKernelGGL(mix_merge_kernel, dim3((unsigned)at->heads), dim3(256), 0, c.stream, u, y, *at, partials, plan.S);
  TLHIP_CHECK_LAUNCH(TLHIP_C_MIX_STEP);
}

}  // namespace tlhip

using namespace tlhip;

extern "C" {

int64_t tlhip_window_ring_ld(int64_t dim) {
  for (int64_t d : {32, 64, 96, 128, 192, 256})
    if (dim > 0 && dim <= d) return d;
  return 0;
}
int64_t tlhip_linear_state_bytes(int64_t heads, int64_t dim, int64_t vdim) {
  return 2 * heads * dim * linear_state_ld(vdim) * (int64_t)sizeof(float);
}
int64_t tlhip_mix_partials_bytes(const tlhip_window_attn* at) {
  if (!at || at->heads <= 0) return 0;
  const int S = attn_splits(at);
  return S > 1 ? at->heads * S * (tlhip_window_ring_ld(at->dim) + 2) * (int64_t)sizeof(float) : 0;
}

int tlhip_mix_step(const void* u, void* y, const tlhip_window_attn* at, const tlhip_linear_attn* la,
                   const tlhip_polynorm* pn, int64_t pos, const void* d_pos, void* partials, int64_t partials_bytes) {
  TLHIP_REQUIRE_READY();
  if (!u || !y || !aligned16(u) || (!at && !la && !pn)) return fail(TLHIP_EINVAL, "tlhip_mix_step: bad operands");
  if (pos < 0 || pos > (1 << 30)) return fail(TLHIP_EINVAL, "tlhip_mix_step: bad position");
  if (at)
    if (int rc = check_window_attn(at, "tlhip_mix_step")) return rc;
  if (la)
    if (int rc = check_linear_attn(la, "tlhip_mix_step")) return rc;
  if (pn)
    if (int rc = check_polynorm(pn, "tlhip_mix_step")) return rc;
  if (at && at->ring_rows < at->window && at->ring_rows < pos + 1)
    return fail(TLHIP_EINVAL, "tlhip_mix_step: the key ring is shorter than the window");
  if (tlhip_mix_partials_bytes(at) > (partials ? partials_bytes : 0))
    return fail(TLHIP_EINVAL, "tlhip_mix_step: partials buffer too small");
  const MixPlan plan = make_plan(at, la, pn);
  const int nf = at ? (int)(at->ring_ld + 63) / 64 : 1;
  const float* pu = static_cast<const float*>(u);
  float* py = static_cast<float*>(y);
  float* pp = static_cast<float*>(partials);
#define TLHIP_MIX(NQ, NF) return launch_mix<NQ, NF>(pu, py, at, la, pn, (int)pos, d_pos, pp, plan)
  switch (plan.nq * 8 + nf) {
    case 8 + 1: TLHIP_MIX(1, 1);
    case 8 + 2: TLHIP_MIX(1, 2);
    case 8 + 3: TLHIP_MIX(1, 3);
    case 8 + 4: TLHIP_MIX(1, 4);
    case 16 + 1: TLHIP_MIX(2, 1);
    case 16 + 2: TLHIP_MIX(2, 2);
    case 16 + 3: TLHIP_MIX(2, 3);
    case 16 + 4: TLHIP_MIX(2, 4);
    case 32 + 1: TLHIP_MIX(4, 1);
    case 32 + 2: TLHIP_MIX(4, 2);
    default: return fail(TLHIP_EUNSUPPORTED, "tlhip_mix_step: no kernel for this head size");
  }
#undef TLHIP_MIX
}

}  // extern "C"
