// Mixture-of-experts routing with a softmax or sigmoid router over real and identity experts (gfx950, wave64).
//
//   router_topk     s = softmax(z) over all NE router outputs (fp32); the k largest of s + correction are chosen
//                   (ties: the lower index); the weights are the chosen s, not renormalised.  Outputs beyond the
//                   first E are IDENTITY experts (their output is the token's input itself).  Counts the rows of
//                   every real expert and hands each (token, choice) its rank within its expert.
//                   Sigmoid scores instead of the softmax, and groups of neighbouring outputs of which only the best
//                   few (by the sum of their two largest scores) are open to the choice: RouterRule.
//   router_offsets  exclusive scan of the counts -> row_off [E + 1]
//   router_scatter  expert-major rows: src[row] = token, row_expert[row], inv[t*k + j] = row (-1: identity)
//   expert_rows     one workgroup per expert-major row: y = W_down act(W_gate h, W_up h), any sizes, fp32 sums; act =
//                   silu(g) u or the clamped unit g' sigmoid(alpha g') (u' + 1), g' = min(g, L), u' = clamp(u, -L, L)
//   moe_combine     out[t] = sum_j w[t][j] * (inv >= 0 ? Y[inv] : h[t]) (+ sigmoid(gate[t]) * add[t])   (fp32)
#include "elem.h"

namespace lwc {
namespace {

constexpr int kMaxPerLane = 8;  // router outputs per lane: NE <= 512

// How scores become choices and weights.
struct RouterRule {
  int sigmoid;       // scores = sigmoid(z), else the softmax over all outputs
  int renorm;        // weights = chosen scores / (their sum + floor) * scale, else chosen scores * scale
  float floor, scale;
  int groups, keep;  // groups > 1: NE / groups neighbours each; only the `keep` best groups are open
};

template <int PER>
__global__ void router_topk_kernel(const float* __restrict__ z, const float* __restrict__ corr,
                                   const float* __restrict__ bias, int ldz, RouterRule rule, int NE, int E, int k,
                                   int* __restrict__ ids, float* __restrict__ wts, int* __restrict__ counts,
                                   int* __restrict__ rank, int T) {
  const int t = blockIdx.x * (blockDim.x >> 6) + (threadIdx.x >> 6);
  if (t >= T) return;
  const int lane = threadIdx.x & 63;
  const float* zr = z + (size_t)t * ldz;
  float v[PER], c[PER];
  float m = -INFINITY;
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int e = lane + 64 * i;
    v[i] = e < NE ? zr[e] + (bias ? bias[e] : 0.f) : -INFINITY;
    m = fmaxf(m, v[i]);
  }
  if (rule.sigmoid) {
#pragma unroll
    for (int i = 0; i < PER; ++i) v[i] = lane + 64 * i < NE ? sigmoid_f(v[i]) : 0.f;
  } else {
    m = wave_max(m);
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int e = lane + 64 * i;
      v[i] = e < NE ? expf(v[i] - m) : 0.f;
      sum += v[i];
    }
    sum = wave_sum(sum);
#pragma unroll
    for (int i = 0; i < PER; ++i) v[i] = v[i] / sum;
  }
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int e = lane + 64 * i;
    c[i] = e < NE ? v[i] + (corr ? corr[e] : 0.f) : -INFINITY;
  }
  if (rule.groups > 1) {  // groups' scores: group g's lives in lane g & 63, slot g >> 6
    const int size = NE / rule.groups;
    float gs[PER];
#pragma unroll
    for (int i = 0; i < PER; ++i) gs[i] = -INFINITY;
    for (int g = 0; g < rule.groups; ++g) {
      float a = -INFINITY, b = -INFINITY;  // this lane's two largest of the group, then the wave's
#pragma unroll
      for (int i = 0; i < PER; ++i) {
        const int e = lane + 64 * i;
        if (e >= g * size && e < (g + 1) * size) {
          b = fmaxf(b, fminf(a, c[i]));
          a = fmaxf(a, c[i]);
        }
      }
#pragma unroll
      for (int o = 32; o > 0; o >>= 1) {
        const float oa = __shfl_xor(a, o, 64), ob = __shfl_xor(b, o, 64);
        b = fmaxf(fmaxf(b, ob), fminf(a, oa));
        a = fmaxf(a, oa);
      }
      const float score = size > 1 ? a + b : a;
#pragma unroll
      for (int i = 0; i < PER; ++i)
        if (lane + 64 * i == g) gs[i] = score;
    }
    unsigned open = 0;  // bit i: this lane's output lane + 64 i may be chosen
    for (int j = 0; j < rule.keep; ++j) {
      float best = -INFINITY;
      int bi = 0x7fffffff;
#pragma unroll
      for (int i = 0; i < PER; ++i)
        if (gs[i] > best) best = gs[i], bi = lane + 64 * i;
#pragma unroll
      for (int o = 32; o > 0; o >>= 1) {
        const float ob = __shfl_xor(best, o, 64);
        const int oi = __shfl_xor(bi, o, 64);
        if (ob > best || (ob == best && oi < bi)) best = ob, bi = oi;
      }
#pragma unroll
      for (int i = 0; i < PER; ++i) {
        const int e = lane + 64 * i;
        if (e == bi) gs[i] = -INFINITY;
        if (e >= bi * size && e < (bi + 1) * size) open |= 1u << i;
      }
    }
#pragma unroll
    for (int i = 0; i < PER; ++i)
      if (!((open >> i) & 1u)) c[i] = -INFINITY;
  }
  float chosen = 0.f;
  for (int j = 0; j < k; ++j) {
    float best = -INFINITY;
    int bi = 0x7fffffff;
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int e = lane + 64 * i;
      if (e < NE && (c[i] > best || (c[i] == best && e < bi))) best = c[i], bi = e;
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ob = __shfl_xor(best, o, 64);
      const int oi = __shfl_xor(bi, o, 64);
      if (ob > best || (ob == best && oi < bi)) best = ob, bi = oi;
    }
    // the winner's lane removes it and reports its score
    float sc = 0.f;
#pragma unroll
    for (int i = 0; i < PER; ++i)
      if (lane + 64 * i == bi) sc = v[i], c[i] = -INFINITY;
    sc = wave_sum(sc);
    chosen += sc;
    if (lane == 0) {
      ids[(size_t)t * k + j] = bi;
      wts[(size_t)t * k + j] = sc;
      rank[(size_t)t * k + j] = bi < E ? atomicAdd(counts + bi, 1) : -1;
    }
  }
  if (lane == 0 && (rule.renorm || rule.scale != 1.0f))  // softmax, floor 0: the softmax over the chosen outputs only
    for (int j = 0; j < k; ++j) wts[(size_t)t * k + j] *= rule.scale / (rule.renorm ? chosen + rule.floor : 1.0f);
}

// Few router outputs (NE <= NMAX): one THREAD per token, the scores in registers.
template <int NMAX>
__global__ void router_topk_thread_kernel(const float* __restrict__ z, const float* __restrict__ corr,
                                          const float* __restrict__ bias, int ldz, RouterRule rule, int NE, int E, int k,
                                          int* __restrict__ ids, float* __restrict__ wts, int* __restrict__ counts,
                                          int* __restrict__ rank, int T) {
  const int t0 = blockIdx.x * blockDim.x + threadIdx.x;
  const bool live = t0 < T;  // lanes past the last token go along (wave-wide votes below) and write nothing
  const int t = live ? t0 : T - 1;
  const float* zr = z + (size_t)t * ldz;
  float v[NMAX], c[NMAX];
  float m = -INFINITY;
#pragma unroll
  for (int i = 0; i < NMAX; ++i) {
    v[i] = i < NE ? zr[i] + (bias ? bias[i] : 0.f) : -INFINITY;
    m = fmaxf(m, v[i]);
  }
  if (rule.sigmoid) {
#pragma unroll
    for (int i = 0; i < NMAX; ++i) v[i] = i < NE ? sigmoid_f(v[i]) : 0.f;
  } else {
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < NMAX; ++i) {
      v[i] = i < NE ? expf(v[i] - m) : 0.f;
      sum += v[i];
    }
#pragma unroll
    for (int i = 0; i < NMAX; ++i) v[i] = v[i] / sum;
  }
#pragma unroll
  for (int i = 0; i < NMAX; ++i) c[i] = i < NE ? v[i] + (corr ? corr[i] : 0.f) : -INFINITY;
  if (rule.groups > 1) {
    const int size = NE / rule.groups;
    float gs[NMAX];
#pragma unroll
    for (int g = 0; g < NMAX; ++g) {
      float a = -INFINITY, b = -INFINITY;  // the group's two largest
#pragma unroll
      for (int i = 0; i < NMAX; ++i)
        if (i >= g * size && i < (g + 1) * size) {
          b = fmaxf(b, fminf(a, c[i]));
          a = fmaxf(a, c[i]);
        }
      gs[g] = g < rule.groups ? (size > 1 ? a + b : a) : -INFINITY;
    }
    unsigned open = 0;  // bit i: output i may be chosen
    for (int j = 0; j < rule.keep; ++j) {
      float best = -INFINITY;
      int bg = 0;
#pragma unroll
      for (int g = 0; g < NMAX; ++g)
        if (gs[g] > best) best = gs[g], bg = g;
#pragma unroll
      for (int g = 0; g < NMAX; ++g)
        if (g == bg) gs[g] = -INFINITY;
      open |= ((1u << size) - 1u) << (bg * size);
    }
#pragma unroll
    for (int i = 0; i < NMAX; ++i)
      if (!((open >> i) & 1u)) c[i] = -INFINITY;
  }
  float chosen = 0.f;
  for (int j = 0; j < k; ++j) {
    float best = -INFINITY, sc = 0.f;
    int bi = 0;
#pragma unroll
    for (int i = 0; i < NMAX; ++i)
      if (i < NE && c[i] > best) best = c[i], bi = i, sc = v[i];
#pragma unroll
    for (int i = 0; i < NMAX; ++i)
      if (i == bi) c[i] = -INFINITY;
    chosen += sc;
    if (live) {
      ids[(size_t)t * k + j] = bi;
      wts[(size_t)t * k + j] = sc;
    }
    // one atomic per (wave, expert) instead of one per token: the wave's tokens that chose expert e take
    // consecutive ranks in lane order
    int rk = -1;
    for (int e = 0; e < E; ++e) {
      const unsigned long long m = __ballot(live && bi == e);
      if (m == 0ull) continue;
      const int leader = __ffsll((long long)m) - 1;
      int base = 0;
      if ((int)(threadIdx.x & 63) == leader) base = atomicAdd(counts + e, __popcll(m));
      base = __shfl(base, leader, 64);
      if (live && bi == e) rk = base + __popcll(m & ((1ull << (threadIdx.x & 63)) - 1ull));
    }
    if (live) rank[(size_t)t * k + j] = rk;
  }
  if (live && (rule.renorm || rule.scale != 1.0f))
    for (int j = 0; j < k; ++j) wts[(size_t)t * k + j] *= rule.scale / (rule.renorm ? chosen + rule.floor : 1.0f);
}

__global__ void router_offsets_kernel(const int* __restrict__ counts, int E, int* __restrict__ row_off) {
  if (threadIdx.x == 0 && blockIdx.x == 0) {
    int o = 0;
    for (int e = 0; e < E; ++e) {
      row_off[e] = o;
      o += counts[e];
    }
    row_off[E] = o;
  }
}

__global__ void router_scatter_kernel(const int* __restrict__ ids, const int* __restrict__ rank,
                                      const int* __restrict__ row_off, int E, int k, int* __restrict__ src,
                                      int* __restrict__ row_expert, int* __restrict__ inv, int total) {
  const int e = blockIdx.x * blockDim.x + threadIdx.x;
  if (e >= total) return;
  const int x = ids[e];
  if (x < E) {
    const int row = row_off[x] + rank[e];
    src[row] = e / k;
    row_expert[row] = x;
    inv[e] = row;
  } else {
    inv[e] = -1;
  }
}

// W_gu [E][2 ff][d]: gate rows then up rows; W_down [E][d][ff]
template <typename AT>
__global__ void __launch_bounds__(256) expert_rows_kernel(const AT* __restrict__ h, int ldh, const int* __restrict__ src,
                                                           const int* __restrict__ row_expert,
                                                           const int* __restrict__ row_off, int E,
                                                           const AT* __restrict__ w_gu, const AT* __restrict__ w_down,
                                                           float* __restrict__ Y, int d, int ff, int clamped, float alpha,
                                                           float limit) {
  extern __shared__ float smem[];  // h [d] | act [ff]
  const int row = blockIdx.x;
  if (row >= row_off[E]) return;
  float* hs = smem;
  float* act = smem + d;
  const int t = src[row], e = row_expert[row];
  for (int i = threadIdx.x; i < d; i += blockDim.x) hs[i] = Elem<AT>::ld(h + (size_t)t * ldh + i);
  __syncthreads();
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, nw = blockDim.x >> 6;
  const AT* wg = w_gu + (size_t)e * 2 * ff * d;
  for (int f = wv; f < ff; f += nw) {
    const AT* g = wg + (size_t)f * d;
    const AT* u = wg + (size_t)(ff + f) * d;
    float sg = 0.f, su = 0.f;
    for (int i = lane; i < d; i += 64) {
      sg += Elem<AT>::ld(g + i) * hs[i];
      su += Elem<AT>::ld(u + i) * hs[i];
    }
    sg = wave_sum(sg);
    su = wave_sum(su);
    if (lane == 0) {
      if (clamped) {
        const float gc = fminf(sg, limit);
        act[f] = gc * sigmoid_f(alpha * gc) * (fminf(fmaxf(su, -limit), limit) + 1.0f);
      } else {
        act[f] = silu_f(sg) * su;
      }
    }
  }
  __syncthreads();
  const AT* wd = w_down + (size_t)e * d * ff;
  for (int c = wv; c < d; c += nw) {
    const AT* r = wd + (size_t)c * ff;
    float s = 0.f;
    for (int i = lane; i < ff; i += 64) s += Elem<AT>::ld(r + i) * act[i];
    s = wave_sum(s);
    if (lane == 0) Y[(size_t)row * d + c] = s;
  }
}

template <typename AT, typename YT>
__global__ void moe_combine_kernel(const YT* __restrict__ Y, const int* __restrict__ inv, const float* __restrict__ wts,
                                   const AT* __restrict__ h, int ldh, int k, float* __restrict__ out, int d,
                                   const AT* __restrict__ add, int lda, const float* __restrict__ gate, int ldg) {
  const int t = blockIdx.x;
  const float ga = gate ? sigmoid_f(gate[(size_t)t * ldg]) : 1.0f;
  for (int c = threadIdx.x; c < d; c += blockDim.x) {
    float s = add ? Elem<AT>::ld(add + (size_t)t * lda + c) * ga : 0.f;
    for (int j = 0; j < k; ++j) {
      const int r = inv[(size_t)t * k + j];
      const float v = r >= 0 ? Elem<YT>::ld(Y + (size_t)r * d + c) : Elem<AT>::ld(h + (size_t)t * ldh + c);
      s += wts[(size_t)t * k + j] * v;
    }
    out[(size_t)t * d + c] = s;
  }
}

// four columns per thread (d a multiple of four, aligned bases)
template <typename AT, typename YT>
__global__ void moe_combine_vec_kernel(const YT* __restrict__ Y, const int* __restrict__ inv, const float* __restrict__ wts,
                                       const AT* __restrict__ h, int ldh, int k, float* __restrict__ out, int d,
                                       const AT* __restrict__ add, int lda, const float* __restrict__ gate, int ldg) {
  const int t = blockIdx.x;
  const float ga = gate ? sigmoid_f(gate[(size_t)t * ldg]) : 1.0f;
  for (int c = threadIdx.x * 4; c < d; c += blockDim.x * 4) {
    float4v s = add ? Vec4<AT>::ld(add + (size_t)t * lda + c) * ga : float4v{0.f, 0.f, 0.f, 0.f};
    for (int j = 0; j < k; ++j) {
      const int r = inv[(size_t)t * k + j];
      const float4v v = r >= 0 ? Vec4<YT>::ld(Y + (size_t)r * d + c) : Vec4<AT>::ld(h + (size_t)t * ldh + c);
      s += v * wts[(size_t)t * k + j];
    }
    Vec4<float>::st(out + (size_t)t * d + c, s);
  }
}

}  // namespace
}  // namespace lwc

using namespace lwc;

extern "C" int r32_router_max_outputs() { return 64 * kMaxPerLane; }

// counts must be zero on entry (E ints)
// z rows have leading dimension ldz; corr (added to the scores for the choice only) and bias (added to the logits) may be
// null; sigmoid, renorm, floor, scale, groups, keep: RouterRule
extern "C" int r32_router(const float* z, int ldz, const float* corr, const float* bias, int sigmoid, int renorm, float floor,
                          float scale, int groups, int keep, int T, int NE, int E, int k,
                          int* ids, float* wts, int* counts, int* rank, int* row_off, int* src, int* row_expert, int* inv,
                          hipStream_t s) {
  if (T <= 0) return 0;
  if (NE > 64 * kMaxPerLane || k < 1 || k > NE || E > NE) return -1;
  if (groups > 1 && (NE % groups != 0 || keep < 1 || keep > groups || k > keep * (NE / groups))) return -1;
  const RouterRule rule{sigmoid, renorm, floor, scale, groups, keep};
  if (NE <= 16) router_topk_thread_kernel<16><<<(T + 63) / 64, 64, 0, s>>>(z, corr, bias, ldz, rule, NE, E, k, ids, wts, counts, rank, T);
  else if (NE <= 64) router_topk_kernel<1><<<(T + 3) / 4, 256, 0, s>>>(z, corr, bias, ldz, rule, NE, E, k, ids, wts, counts, rank, T);
  else router_topk_kernel<kMaxPerLane><<<(T + 3) / 4, 256, 0, s>>>(z, corr, bias, ldz, rule, NE, E, k, ids, wts, counts, rank, T);
  router_offsets_kernel<<<1, 64, 0, s>>>(counts, E, row_off);
  const int total = T * k;
  router_scatter_kernel<<<(total + 255) / 256, 256, 0, s>>>(ids, rank, row_off, E, k, src, row_expert, inv, total);
  LWC_CHECK_LAUNCH();
  return 0;
}

extern "C" int r32_expert_rows(const void* h, int ldh, const int* src, const int* row_expert, const int* row_off, int E,
                               const void* w_gu, const void* w_down, float* Y, int rows, int d, int ff, int clamped, float alpha,
                               float limit, int f32, hipStream_t s) {
  if (rows <= 0) return 0;
  const size_t shm = (size_t)(d + ff) * sizeof(float);
  if (shm > 60000) return -1;
  if (f32)
    expert_rows_kernel<float><<<rows, 256, shm, s>>>((const float*)h, ldh, src, row_expert, row_off, E, (const float*)w_gu,
                                                      (const float*)w_down, Y, d, ff, clamped, alpha, limit);
  else
    expert_rows_kernel<bf16_t><<<rows, 256, shm, s>>>((const bf16_t*)h, ldh, src, row_expert, row_off, E, (const bf16_t*)w_gu,
                                                       (const bf16_t*)w_down, Y, d, ff, clamped, alpha, limit);
  LWC_CHECK_LAUNCH();
  return 0;
}

// add: rows of the activation type added to every token's sum (a shared expert), or null; gate: fp32 logits, one per
// token (stride ldg), whose sigmoid multiplies the added row, or null
extern "C" int r32_moe_combine(const void* Y, int y_f32, const int* inv, const float* wts, const void* h, int ldh, int T,
                               int k, float* out, int d, const void* add, int lda, const float* gate, int ldg, int f32,
                               hipStream_t s) {
  if (T <= 0) return 0;
  if (d % 4 == 0 && ldh % 4 == 0 && lda % 4 == 0 && aligned_to(add, f32 ? 16 : 8) && aligned_to(Y, y_f32 ? 16 : 8) && aligned_to(h, f32 ? 16 : 8) && aligned_to(out, 16)) {
    if (f32 && y_f32)
      moe_combine_vec_kernel<float, float><<<T, 256, 0, s>>>((const float*)Y, inv, wts, (const float*)h, ldh, k, out, d, (const float*)add, lda, gate, ldg);
    else if (!f32 && y_f32)
      moe_combine_vec_kernel<bf16_t, float><<<T, 256, 0, s>>>((const float*)Y, inv, wts, (const bf16_t*)h, ldh, k, out, d, (const bf16_t*)add, lda, gate, ldg);
    else if (!f32 && !y_f32)
      moe_combine_vec_kernel<bf16_t, bf16_t><<<T, 256, 0, s>>>((const bf16_t*)Y, inv, wts, (const bf16_t*)h, ldh, k, out, d, (const bf16_t*)add, lda, gate, ldg);
    else
      return -1;
    LWC_CHECK_LAUNCH();
    return 0;
  }
  if (f32 && y_f32)
    moe_combine_kernel<float, float><<<T, 256, 0, s>>>((const float*)Y, inv, wts, (const float*)h, ldh, k, out, d, (const float*)add, lda, gate, ldg);
  else if (!f32 && y_f32)
    moe_combine_kernel<bf16_t, float><<<T, 256, 0, s>>>((const float*)Y, inv, wts, (const bf16_t*)h, ldh, k, out, d, (const bf16_t*)add, lda, gate, ldg);
  else if (!f32 && !y_f32)
    moe_combine_kernel<bf16_t, bf16_t><<<T, 256, 0, s>>>((const bf16_t*)Y, inv, wts, (const bf16_t*)h, ldh, k, out, d, (const bf16_t*)add, lda, gate, ldg);
  else
    return -1;
  LWC_CHECK_LAUNCH();
  return 0;
}
