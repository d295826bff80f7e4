// Sublayers whose norm comes AFTER the residual sum (gfx950, wave64): x <- rms_norm(alpha x + y) * w on the fp32 stream.
//
//   post_norm          y = one row per token (bf16 or fp32)
//   post_norm_experts  y = a routed feed-forward, formed on the way: sum_j w[t][j] Y[inv[t k + j]] (expert-major rows)
//                      + sigmoid(gate[t]) * shared[t]; the sum never goes to memory
// Both also write the new x as bf16 rows, the next sublayer's input (it reads x itself).  Statistics are fp32.
#include "elem.h"

namespace lwc {
namespace {

template <typename YT>
__global__ void post_norm_kernel(float* __restrict__ x, const YT* __restrict__ y, int ldy, float alpha,
                                 const float* __restrict__ w, bf16_t* __restrict__ cast, int d, float eps) {
  __shared__ float scratch[16];
  const int t = blockIdx.x;
  float* xr = x + (size_t)t * d;
  float s = 0.f;
  for (int i = threadIdx.x; i < d; i += blockDim.x) {
    const float v = alpha * xr[i] + Elem<YT>::ld(y + (size_t)t * ldy + i);
    xr[i] = v;  // (each thread re-reads only what it wrote)
    s += v * v;
  }
  const float rstd = 1.0f / sqrtf(block_sum(s, scratch) / (float)d + eps);
  for (int i = threadIdx.x; i < d; i += blockDim.x) {
    const float v = xr[i] * rstd * w[i];
    xr[i] = v;
    if (cast) cast[(size_t)t * d + i] = f2bf(v);
  }
}

// The sum stays in registers between the statistics and the write: rows of d <= 1024 NCH entries, bases a multiple of
// four entries.
template <int NCH>
LWC_DEVICE void norm_and_store(float4v (&v)[NCH], float s, float* scratch, float* xr, const float* w, bf16_t* cr, int d, float eps) {
  const float rstd = 1.0f / sqrtf(block_sum(s, scratch) / (float)d + eps);
#pragma unroll
  for (int u = 0; u < NCH; ++u) {
    const int i = (threadIdx.x + 256 * u) * 4;
    if (i < d) {
      const float4v o = v[u] * rstd * Vec4<float>::ld(w + i);
      Vec4<float>::st(xr + i, o);
      if (cr) Vec4<bf16_t>::st(cr + i, o);
    }
  }
}

template <typename YT, int NCH>
__global__ void __launch_bounds__(256) post_norm_vec_kernel(float* __restrict__ x, const YT* __restrict__ y, int ldy, float alpha,
                                                             const float* __restrict__ w, bf16_t* __restrict__ cast, int d,
                                                             float eps) {
  __shared__ float scratch[16];
  const int t = blockIdx.x;
  float* xr = x + (size_t)t * d;
  float4v v[NCH];
  float s = 0.f;
#pragma unroll
  for (int u = 0; u < NCH; ++u) {
    const int i = (threadIdx.x + 256 * u) * 4;
    v[u] = float4v{0.f, 0.f, 0.f, 0.f};
    if (i < d) {
      v[u] = Vec4<float>::ld(xr + i) * alpha + Vec4<YT>::ld(y + (size_t)t * ldy + i);
      s += v[u][0] * v[u][0] + v[u][1] * v[u][1] + v[u][2] * v[u][2] + v[u][3] * v[u][3];
    }
  }
  norm_and_store<NCH>(v, s, scratch, xr, w, cast ? cast + (size_t)t * d : nullptr, d, eps);
}

// YT: the experts' rows, AT: the shared expert's (may be null: none)
template <typename YT, typename AT, int NCH>
__global__ void __launch_bounds__(256) post_norm_experts_kernel(float* __restrict__ x, const YT* __restrict__ Y,
                                                                 const int* __restrict__ inv, const float* __restrict__ wts, int k,
                                                                 const AT* __restrict__ shared, int lds,
                                                                 const float* __restrict__ gate, int ldg, float alpha,
                                                                 const float* __restrict__ w, bf16_t* __restrict__ cast, int d,
                                                                 float eps) {
  __shared__ float scratch[16];
  const int t = blockIdx.x;
  float* xr = x + (size_t)t * d;
  float4v v[NCH];
  const float gs = shared ? (gate ? sigmoid_f(gate[(size_t)t * ldg]) : 1.0f) : 0.f;
#pragma unroll
  for (int u = 0; u < NCH; ++u) {
    const int i = (threadIdx.x + 256 * u) * 4;
    v[u] = float4v{0.f, 0.f, 0.f, 0.f};
    if (i < d) {
      v[u] = Vec4<float>::ld(xr + i) * alpha;
      if (shared) v[u] += Vec4<AT>::ld(shared + (size_t)t * lds + i) * gs;
    }
  }
  for (int j = 0; j < k; ++j) {
    const int r = inv[(size_t)t * k + j];
    if (r < 0) continue;  // (a choice without a row)
    const float wj = wts[(size_t)t * k + j];
    const YT* yr = Y + (size_t)r * d;
#pragma unroll
    for (int u = 0; u < NCH; ++u) {
      const int i = (threadIdx.x + 256 * u) * 4;
      if (i < d) v[u] += Vec4<YT>::ld(yr + i) * wj;
    }
  }
  float s = 0.f;
#pragma unroll
  for (int u = 0; u < NCH; ++u) s += v[u][0] * v[u][0] + v[u][1] * v[u][1] + v[u][2] * v[u][2] + v[u][3] * v[u][3];
  norm_and_store<NCH>(v, s, scratch, xr, w, cast ? cast + (size_t)t * d : nullptr, d, eps);
}

}  // namespace
}  // namespace lwc

using namespace lwc;

extern "C" int r32_post_norm(float* x, const void* y, int ldy, float alpha, const float* w, void* cast, int T, int d, float eps,
                             int y_f32, hipStream_t s) {
  if (T <= 0) return 0;
  const bool vec = d % 4 == 0 && d <= 8192 && ldy % 4 == 0 && aligned_to(x, 16) && aligned_to(w, 16) &&
                   aligned_to(y, y_f32 ? 16 : 8) && aligned_to(cast, 8);
  const int nch = (d + 1023) / 1024;
  bf16_t* c = (bf16_t*)cast;
#define LWC_PN(YT)                                                                                             \
  if (!vec) post_norm_kernel<YT><<<T, 256, 0, s>>>(x, (const YT*)y, ldy, alpha, w, c, d, eps);                 \
  else if (nch <= 1) post_norm_vec_kernel<YT, 1><<<T, 256, 0, s>>>(x, (const YT*)y, ldy, alpha, w, c, d, eps); \
  else if (nch <= 2) post_norm_vec_kernel<YT, 2><<<T, 256, 0, s>>>(x, (const YT*)y, ldy, alpha, w, c, d, eps); \
  else if (nch <= 4) post_norm_vec_kernel<YT, 4><<<T, 256, 0, s>>>(x, (const YT*)y, ldy, alpha, w, c, d, eps); \
  else post_norm_vec_kernel<YT, 8><<<T, 256, 0, s>>>(x, (const YT*)y, ldy, alpha, w, c, d, eps)
  if (y_f32) {
    LWC_PN(float);
  } else {
    LWC_PN(bf16_t);
  }
#undef LWC_PN
  LWC_CHECK_LAUNCH();
  return 0;
}

// Whether post_norm_experts takes rows of d entries (else: moe_combine, then post_norm).
extern "C" int r32_post_norm_experts_ok(int d) { return d % 4 == 0 && d <= 8192; }

// io: bit 0 = Y fp32 (else bf16), bit 1 = shared fp32 (else bf16); shared and gate may be null.
extern "C" int r32_post_norm_experts(float* x, const void* Y, const int* inv, const float* wts, int k, const void* shared, int lds,
                                     const float* gate, int ldg, float alpha, const float* w, void* cast, int T, int d, float eps,
                                     int io, hipStream_t s) {
  if (T <= 0) return 0;
  const bool yf = io & 1, sf = io & 2;
  if (!r32_post_norm_experts_ok(d) || lds % 4 != 0 || !aligned_to(x, 16) || !aligned_to(w, 16) || !aligned_to(Y, yf ? 16 : 8) ||
      !aligned_to(shared, sf ? 16 : 8) || !aligned_to(cast, 8))
    return -1;
  const int nch = (d + 1023) / 1024;
  bf16_t* c = (bf16_t*)cast;
#define LWC_PNE2(YT, AT, N)                                                                                                  \
  post_norm_experts_kernel<YT, AT, N><<<T, 256, 0, s>>>(x, (const YT*)Y, inv, wts, k, (const AT*)shared, lds, gate, ldg, alpha, \
                                                        w, c, d, eps)
#define LWC_PNE(YT, AT)                  \
  if (nch <= 1) LWC_PNE2(YT, AT, 1);     \
  else if (nch <= 2) LWC_PNE2(YT, AT, 2); \
  else if (nch <= 4) LWC_PNE2(YT, AT, 4); \
  else LWC_PNE2(YT, AT, 8)
  if (yf && sf) {
    LWC_PNE(float, float);
  } else if (yf) {
    LWC_PNE(float, bf16_t);
  } else if (!sf) {
    LWC_PNE(bf16_t, bf16_t);
  } else {
    return -1;
  }
#undef LWC_PNE
#undef LWC_PNE2
  LWC_CHECK_LAUNCH();
  return 0;
}
