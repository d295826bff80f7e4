// Parallel residual streams mixed at every sublayer ("hyper-connections"), with the elementwise bounded norm
//   dyt(x) = tanh(a x) * w + b        (a: one number, w and b: one per column; no statistics)
// in front of each sublayer (gfx950, wave64).  The S streams are fp32 planes X [S, T, d].
//
//   embed_streams   x = dyt_e(table[token] * scale);  X_s = x for every s;  h = dyt(sum_s in_s x)
//   hyper_step      behind a sublayer with result y (+ a bias per column):
//                     X'_t = sum_s mix[s][t] X_s + out[t] (y + bias)      all streams from the old ones
//                     u    = sum_t in[t] X'_t                             the NEXT sublayer's input (ones: the streams' sum)
//                     h    = dyt(u)                                       rows of the activation type
//                   X' overwrites X, or stays unwritten (the last sublayer, whose streams nobody reads); with a row list
//                   only these rows are formed (h row n = token rows[n], y row too) and X stays as it is.
// Coefficients of one step, fp32: [ mix (S x S, from-major) | out (S) | in (S) ].  Everything is elementwise over the
// columns, so a step reads and writes every stream once.
#include "elem.h"

namespace lwc {
namespace {

// tanh for rows of the activation type.  bf16 rows: 1 - 2 / (exp(2 x) + 1), absolute error ~1e-7, far below the rounding of
// the result; fp32 rows: tanhf.
template <typename AT> LWC_DEVICE float tanh_rows(float x) { return tanhf(x); }
template <> LWC_DEVICE float tanh_rows<bf16_t>(float x) { return 1.0f - 2.0f * __builtin_amdgcn_rcpf(__expf(2.0f * x) + 1.0f); }

template <typename AT> LWC_DEVICE float dyt1(float x, float a, float w, float b) { return tanh_rows<AT>(a * x) * w + b; }
template <typename AT> LWC_DEVICE float4v dyt4(float4v x, float a, float4v w, float4v b) {
  return float4v{dyt1<AT>(x[0], a, w[0], b[0]), dyt1<AT>(x[1], a, w[1], b[1]), dyt1<AT>(x[2], a, w[2], b[2]),
                 dyt1<AT>(x[3], a, w[3], b[3])};
}

struct HyperParams {
  float* X;             // [S, T, d]
  long long plane;      // T * d
  int S;
  const void* y;        // [T, d], or `parts` such planes whose sum is the result (the partial products of a split GEMM)
  int ldy, parts;
  long long ypart;      // between the planes
  const float* bias;    // [d] or null
  const float* coef;    // [S*S | S | S]
  float a;
  const float* w;
  const float* b;
  void* h;              // [n, d], n = T or the row list's length
  const long long* rows;
  int n, d, write;
};

// NS: the stream count when EXACT, else its upper bound (streams beyond S are skipped)
template <typename YT, typename AT, int NS, bool EXACT>
__global__ void __launch_bounds__(256) hyper_step_vec_kernel(const HyperParams p) {
  const int c = 4 * (blockIdx.x * blockDim.x + threadIdx.x);
  if (c >= p.d) return;
  const int S = EXACT ? NS : p.S;
  const float* mix = p.coef;
  const float* out = p.coef + S * S;
  const float* in = out + S;
  const float4v w = Vec4<float>::ld(p.w + c), b = Vec4<float>::ld(p.b + c);
  const float4v bias = p.bias ? Vec4<float>::ld(p.bias + c) : float4v{0.f, 0.f, 0.f, 0.f};
  for (int r = blockIdx.y; r < p.n; r += gridDim.y) {
    const long long t = p.rows ? p.rows[r] : r;
    float* xr = p.X + t * p.d + c;
    float4v y = Vec4<YT>::ld((const YT*)p.y + t * p.ldy + c) + bias;
    for (int k = 1; k < p.parts; ++k) y += Vec4<YT>::ld((const YT*)p.y + k * p.ypart + t * p.ldy + c);
    float4v x[NS];
#pragma unroll
    for (int s = 0; s < NS; ++s)
      if (EXACT || s < S) x[s] = Vec4<float>::ld(xr + s * p.plane);
    float4v u = float4v{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int q = 0; q < NS; ++q) {
      if (EXACT || q < S) {
        float4v v = y * out[q];
#pragma unroll
        for (int s = 0; s < NS; ++s)
          if (EXACT || s < S) v += x[s] * mix[s * S + q];
        u += v * in[q];
        if (p.write) Vec4<float>::st(xr + q * p.plane, v);
      }
    }
    Vec4<AT>::st((AT*)p.h + (size_t)r * p.d + c, dyt4<AT>(u, p.a, w, b));
  }
}

template <typename YT, typename AT, int NS>
__global__ void __launch_bounds__(256) hyper_step_kernel(const HyperParams p) {
  const int c = blockIdx.x * blockDim.x + threadIdx.x;
  if (c >= p.d) return;
  const int S = p.S;
  const float* mix = p.coef;
  const float* out = p.coef + S * S;
  const float* in = out + S;
  for (int r = blockIdx.y; r < p.n; r += gridDim.y) {
    const long long t = p.rows ? p.rows[r] : r;
    float* xr = p.X + t * p.d + c;
    float y = Elem<YT>::ld((const YT*)p.y + t * p.ldy + c) + (p.bias ? p.bias[c] : 0.f);
    for (int k = 1; k < p.parts; ++k) y += Elem<YT>::ld((const YT*)p.y + k * p.ypart + t * p.ldy + c);
    float x[NS];
#pragma unroll
    for (int s = 0; s < NS; ++s) x[s] = s < S ? xr[s * p.plane] : 0.f;
    float u = 0.f;
#pragma unroll
    for (int q = 0; q < NS; ++q) {
      if (q < S) {
        float v = y * out[q];
#pragma unroll
        for (int s = 0; s < NS; ++s)
          if (s < S) v += x[s] * mix[s * S + q];
        u += v * in[q];
        if (p.write) xr[q * p.plane] = v;
      }
    }
    Elem<AT>::st((AT*)p.h + (size_t)r * p.d + c, dyt1<AT>(u, p.a, p.w[c], p.b[c]));
  }
}

template <typename TT, typename AT>
__global__ void __launch_bounds__(256) embed_streams_kernel(const TT* __restrict__ table, const int* __restrict__ tokens, int vocab,
                                                             float scale, float ae, const float* __restrict__ we,
                                                             const float* __restrict__ be, const float* __restrict__ in, int S,
                                                             float a, const float* __restrict__ w, const float* __restrict__ b,
                                                             float* __restrict__ X, AT* __restrict__ h, int T, int d) {
  const int t = blockIdx.x;
  int tok = tokens[t];
  tok = tok < 0 ? 0 : (tok >= vocab ? vocab - 1 : tok);
  const TT* row = table + (size_t)tok * d;
  const long long plane = (long long)T * d;
  float g = 0.f;
  for (int s = 0; s < S; ++s) g += in[s];
  for (int i = blockIdx.y * blockDim.x + threadIdx.x; i < d; i += gridDim.y * blockDim.x) {
    const float x = dyt1<float>(Elem<TT>::ld(row + i) * scale, ae, we[i], be[i]);
    for (int s = 0; s < S; ++s) X[s * plane + (size_t)t * d + i] = x;
    Elem<AT>::st(h + (size_t)t * d + i, dyt1<AT>(x * g, a, w[i], b[i]));
  }
}

template <typename YT, typename AT>
void launch_hyper(const HyperParams& p, bool vec, hipStream_t s) {
  const int units = vec ? p.d / 4 : p.d, bx = (units + 255) / 256;
  int by = 16384 / bx;  // a thread keeps its columns' weights over several rows
  by = by < 1 ? 1 : by;
  const dim3 grid(bx, p.n < by ? p.n : by);
  if (vec) {
    switch (p.S) {
      case 1: hyper_step_vec_kernel<YT, AT, 1, true><<<grid, 256, 0, s>>>(p); break;
      case 2: hyper_step_vec_kernel<YT, AT, 2, true><<<grid, 256, 0, s>>>(p); break;
      case 3: hyper_step_vec_kernel<YT, AT, 3, true><<<grid, 256, 0, s>>>(p); break;
      case 4: hyper_step_vec_kernel<YT, AT, 4, true><<<grid, 256, 0, s>>>(p); break;
      default:
        if (p.S <= 8) hyper_step_vec_kernel<YT, AT, 8, false><<<grid, 256, 0, s>>>(p);
        else hyper_step_vec_kernel<YT, AT, 16, false><<<grid, 256, 0, s>>>(p);
    }
  } else if (p.S <= 4) {
    hyper_step_kernel<YT, AT, 4><<<grid, 256, 0, s>>>(p);
  } else {
    hyper_step_kernel<YT, AT, 16><<<grid, 256, 0, s>>>(p);
  }
}

}  // namespace
}  // namespace lwc

using namespace lwc;

extern "C" int r32_hyper_max_streams() { return 16; }

// io: bit 0 = table fp32 (else bf16), bit 1 = h fp32 (else bf16)
extern "C" int r32_embed_streams(const void* table, const int* tokens, int vocab, float scale, float ae, const float* we,
                                 const float* be, const float* in, int S, float a, const float* w, const float* b, float* X,
                                 void* h, int T, int d, int io, hipStream_t s) {
  if (T <= 0) return 0;
  if (S < 1 || S > r32_hyper_max_streams()) return -1;
  const int parts = (d + 255) / 256;
  const dim3 grid(T, T >= 1024 ? 1 : (parts < 16 ? parts : 16));  // few rows: several workgroups per row
  if (io == 3)
    embed_streams_kernel<float, float><<<grid, 256, 0, s>>>((const float*)table, tokens, vocab, scale, ae, we, be, in, S, a, w, b, X,
                                                         (float*)h, T, d);
  else if (io == 0)
    embed_streams_kernel<bf16_t, bf16_t><<<grid, 256, 0, s>>>((const bf16_t*)table, tokens, vocab, scale, ae, we, be, in, S, a, w, b,
                                                           X, (bf16_t*)h, T, d);
  else
    return -1;
  LWC_CHECK_LAUNCH();
  return 0;
}

// io: bit 0 = y fp32 (else bf16), bit 1 = h fp32 (else bf16)
extern "C" int r32_hyper_step(float* X, long long plane, int S, const void* y, int ldy, int parts, long long ypart, const float* bias,
                              const float* coef, float a, const float* w, const float* b, void* h, const long long* rows, int n, int d, int write, int io,
                              hipStream_t s) {
  if (n <= 0) return 0;
  if (S < 1 || S > r32_hyper_max_streams() || (write && rows) || parts < 1) return -1;
  HyperParams p;
  p.X = X; p.plane = plane; p.S = S; p.y = y; p.ldy = ldy; p.parts = parts; p.ypart = ypart; p.bias = bias; p.coef = coef; p.a = a; p.w = w; p.b = b; p.h = h;
  p.rows = rows; p.n = n; p.d = d; p.write = write;
  const bool yf = io & 1, hf = io & 2;
  const bool vec = d % 4 == 0 && ldy % 4 == 0 && ypart % 4 == 0 && plane % 4 == 0 && aligned_to(X, 16) && aligned_to(y, yf ? 16 : 8) &&
                   aligned_to(bias, 16) && aligned_to(w, 16) && aligned_to(b, 16) && aligned_to(h, hf ? 16 : 8);
  if (yf && hf) launch_hyper<float, float>(p, vec, s);
  else if (!yf && !hf) launch_hyper<bf16_t, bf16_t>(p, vec, s);
  else if (yf) launch_hyper<float, bf16_t>(p, vec, s);
  else return -1;
  LWC_CHECK_LAUNCH();
  return 0;
}
