// Expert choice of one token from its router logits, shared by the kernels that route (seqmix.hip, mix_sandwich.hip).
//
//   scores    s = softmax(z) over the experts, or sigmoid(z) expert by expert;
//   choice    c = s + bias (bias may be null); experts outside the `keep` best of G equal groups of neighbours are out, a group's score
//             being the sum of its `group_best` largest choice scores (1 or 2; a group of one expert has one); the `top` largest choice
//             scores win (ties: the lower index); choice scores may be negative, so what is out counts as minus infinity;
//   weights   w_k = s_k / (sum of the chosen s + 1e-20) * scale.
// Everything in fp32, sums in a fixed order: the result depends on the logits only.
#ifndef MSGL_MIX_ROUTE_H_
#define MSGL_MIX_ROUTE_H_

#include "mix_common.h"

namespace {

struct RouteRule {
  int sigmoid;     // scores: 0 softmax, 1 sigmoid
  int group_best;  // 1 or 2
  float scale;
};

__device__ __forceinline__ float group_score(const float* c, int per, int group_best) {
  float a = -INFINITY, b = -INFINITY;  // the largest and the second largest
  for (int e = 0; e < per; ++e) {
    const float v = c[e];
    if (v > a) {
      b = a;
      a = v;
    } else {
      b = fmaxf(b, v);
    }
  }
  return group_best == 2 && per > 1 ? a + b : a;
}

__device__ __forceinline__ float wave_max_f(float v) {
#pragma unroll
  for (int o = 32; o >= 1; o >>= 1) v = fmaxf(v, __shfl_xor(v, o, 64));
  return v;
}

// The 64 lanes of one wave over one token (lane owns experts lane, lane + 64, ...).  s: the E logits on entry; s, c: E entries of LDS each,
// gs: G + top.
template <typename T>
__device__ __forceinline__ void select_experts_wave(float* s, float* c, float* gs, const T* __restrict__ bias, int E, int top, int G,
                                                    int keep, RouteRule rule, int* __restrict__ ids, float* __restrict__ wts) {
  const int lane = threadIdx.x & 63;
  if (rule.sigmoid) {
    for (int e = lane; e < E; e += 64) {
      const float v = 1.0f / (1.0f + expf(-s[e]));
      s[e] = v;
      c[e] = v + (bias ? ld(bias + e) : 0.f);
    }
  } else {
    float mx = -INFINITY;
    for (int e = lane; e < E; e += 64) mx = fmaxf(mx, s[e]);
    mx = wave_max_f(mx);
    float sum = 0.f;
    for (int e = lane; e < E; e += 64) {
      const float v = expf(s[e] - mx);
      s[e] = v;
      sum += v;
    }
    sum = wave_sum(sum);
    for (int e = lane; e < E; e += 64) {
      const float v = s[e] / sum;
      s[e] = v;
      c[e] = v + (bias ? ld(bias + e) : 0.f);
    }
  }
  const int per = E / G;
  if (keep < G) {
    for (int g = lane; g < G; g += 64) gs[g] = group_score(c + g * per, per, rule.group_best);
    for (int g = lane; g < G; g += 64) {
      const float mine = gs[g];
      int better = 0;
      for (int o2 = 0; o2 < G; ++o2) better += (gs[o2] > mine) || (gs[o2] == mine && o2 < g);
      if (better >= keep)
        for (int e = g * per; e < (g + 1) * per; ++e) c[e] = -INFINITY;
    }
  }
  float tot = 0.f;
  for (int k = 0; k < top; ++k) {
    float bv = -INFINITY;
    int best = 0x7fffffff;
    for (int e = lane; e < E; e += 64) {
      const float v = c[e];
      if (v > bv) {
        bv = v;
        best = e;
      }
    }
#pragma unroll
    for (int o = 32; o >= 1; o >>= 1) {
      const float ov = __shfl_xor(bv, o, 64);
      const int oi = __shfl_xor(best, o, 64);
      if (ov > bv || (ov == bv && oi < best)) {
        bv = ov;
        best = oi;
      }
    }
    if (best == 0x7fffffff) best = 0;  // unreachable: the host checks top <= keep * (E / G) and choice scores are finite
    const float sv = s[best];
    tot += sv;
    if (lane == 0) {
      ids[k] = best;
      gs[G + k] = sv;  // the chosen scores wait in LDS (in order within the wave) for the sum
      c[best] = -INFINITY;
    }
  }
  const float inv = rule.scale / (tot + 1e-20f);
  for (int k = lane; k < top; k += 64) wts[k] = gs[G + k] * inv;
}

// Router logits of ONE row by a workgroup of WAVES waves: sc[e] = router[e] . row (row: W fp32 numbers in LDS, as the router reads them; the
// caller has synchronized after writing it and synchronizes before reading sc).  A wave takes experts wave, wave + WAVES, ...; up to kRouteAcc
// of them at once, so that one pass over the row has that many independent weight loads in flight per lane (element order per expert:
// lane-strided, then the wave reduction: fixed).
template <int WAVES, typename T>
__device__ __forceinline__ void router_logits(const float* row, const T* __restrict__ router, int E, int W, float* sc) {
  constexpr int kRouteAcc = 8;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const bool wide = (W & 7) == 0 && ((uintptr_t)router & 15u) == 0;
  for (int e0 = wave; e0 < E; e0 += WAVES * kRouteAcc) {
    float acc[kRouteAcc];
#pragma unroll
    for (int a = 0; a < kRouteAcc; ++a) acc[a] = 0.f;
    if (wide) {  // eight consecutive weights per lane and load: 16 bytes (bf16) or 32 (fp32)
      for (int i = lane * 8; i < W; i += 512) {
        float hv[8];
#pragma unroll
        for (int u = 0; u < 8; ++u) hv[u] = row[i + u];
#pragma unroll
        for (int a = 0; a < kRouteAcc; ++a) {
          const int e = e0 + WAVES * a;
          if (e < E) {
            float wv[8];
            read8(router + (size_t)e * W + i, wv);
#pragma unroll
            for (int u = 0; u < 8; ++u) acc[a] = fmaf(hv[u], wv[u], acc[a]);
          }
        }
      }
    } else {
      for (int i = lane; i < W; i += 64) {
        const float hv = row[i];
#pragma unroll
        for (int a = 0; a < kRouteAcc; ++a) {
          const int e = e0 + WAVES * a;
          if (e < E) acc[a] = fmaf(hv, ld(router + (size_t)e * W + i), acc[a]);
        }
      }
    }
#pragma unroll
    for (int a = 0; a < kRouteAcc; ++a) {
      const int e = e0 + WAVES * a;
      const float v = wave_sum(acc[a]);
      if (e < E && lane == 0) sc[e] = v;
    }
  }
}

}  // namespace

#endif
