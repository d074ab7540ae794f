// Mixture-of-experts pieces for dense (bf16 / fp32) expert weights of any width:
//   * a router with sigmoid scores, an optional selection-only correction and normalised weights,
//     or with biased logits and the softmax over the chosen logits as weights; optionally only experts of
//     the best groups of neighbouring experts can be chosen;
//   * the routed experts of small batches as (token, expert) pair GEMVs: gate|up with the SiLU
//     gating fused (or an ungated up projection with relu squared), then the down projection with the
//     weighted top-k combine fused, no atomics.
// Larger batches group rows by expert and run library GEMMs (the caller's choice).
#include "common.h"

namespace la {

// One wave per token: z_e = router[e] . x (fp32).
// mode 0: s = sigmoid(z); the `topk` largest s + corr are chosen (ties: lowest expert id), their
//         weights are s / (sum of the chosen s + 1e-20).
// mode 1: s = z + corr (a bias that counts in the weights too); the `topk` largest s are chosen,
//         their weights are the softmax over the chosen s.
// groups > 1: experts form that many groups of neighbours; a group's score is its largest s (+ corr), and only
// experts of the `keep` best groups can be chosen (ties: lowest group).  All weights times scale.
// SPREAD (batches of few rows): a workgroup per token whose waves take two experts each at a time, wave 0 chooses.
template <typename AT, bool SPREAD>
__global__ __launch_bounds__(SPREAD ? 1024 : 256) void router_topk_kernel(const AT* __restrict__ x, long ldx,
                                                          const float* __restrict__ router,
                                                          const float* __restrict__ corr, int E, int D, int T,
                                                          int topk, int renorm, int mode, int groups, int keep,
                                                          float scale, int* __restrict__ ids, float* __restrict__ wts) {
  constexpr int NR = SPREAD ? 1 : 4, KE = SPREAD ? 2 : 8;     // tokens a workgroup, experts a pass of a wave
  __shared__ float sc[NR][256];
  __shared__ uint8_t open[NR][256];    // the expert's group can be chosen from
  const int wave = threadIdx.x >> 6, w = SPREAD ? 0 : wave, lane = threadIdx.x & 63;
  const int t = blockIdx.x * NR + w;
  const bool chooses = !SPREAD || wave == 0;
  const bool live = t < T;
  const AT* xr = x + (long)(live ? t : 0) * ldx;
  // KE experts at a time: x is read once per pass and the router rows give independent loads
  for (int e0 = SPREAD ? wave * KE : 0; e0 < E; e0 += SPREAD ? (int)(blockDim.x >> 6) * KE : KE) {
    float a[KE];
#pragma unroll
    for (int k = 0; k < KE; ++k) a[k] = 0.f;
    if ((D & 3) == 0) {
      // U slices of 256 columns at a time, all their loads before the first sum; past the row's end or the last
      // expert: some valid element, times 0 or into a sum nobody reads
      constexpr int U = SPREAD ? 8 : 2;
      for (int d0 = lane * 4; d0 - lane * 4 < D; d0 += 256 * U) {
        AT xv[U][4];
        float4 rv[U][KE];
#pragma unroll
        for (int u = 0; u < U; ++u) {
          const int d = min(d0 + 256 * u, D - 4);
#pragma unroll
          for (int j = 0; j < 4; ++j) xv[u][j] = xr[d + j];
#pragma unroll
          for (int k = 0; k < KE; ++k) rv[u][k] = *(const float4*)(router + (long)min(e0 + k, E - 1) * D + d);
        }
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int u = 0; u < U; ++u) {
          const float in = d0 + 256 * u < D ? 1.f : 0.f;
          const float x0 = in * (float)xv[u][0], x1 = in * (float)xv[u][1], x2 = in * (float)xv[u][2], x3 = in * (float)xv[u][3];
#pragma unroll
          for (int k = 0; k < KE; ++k)
            a[k] = fmaf(rv[u][k].x, x0, fmaf(rv[u][k].y, x1, fmaf(rv[u][k].z, x2, fmaf(rv[u][k].w, x3, a[k]))));
        }
      }
    } else {
      for (int d = lane; d < D; d += 64) {
        const float xv = (float)xr[d];
#pragma unroll
        for (int k = 0; k < KE; ++k)
          if (e0 + k < E) a[k] = fmaf(router[(long)(e0 + k) * D + d], xv, a[k]);
      }
    }
#pragma unroll
    for (int k = 0; k < KE; ++k) {
      const float v = wave_sum(a[k]);
      if (lane == 0 && e0 + k < E) sc[w][e0 + k] = mode ? v + (corr ? corr[e0 + k] : 0.f) : 1.f / (1.f + __expf(-v));
    }
  }
  __syncthreads();
  if (groups > 1 && chooses) {
    const int n = E / groups;
    float gm[4];                       // scores of groups lane, lane + 64, ..
    for (int i = 0; i < 4; ++i) {
      const int g = lane + 64 * i;
      gm[i] = -INFINITY;
      if (g < groups)
        for (int e = g * n; e < (g + 1) * n; ++e) {
          gm[i] = fmaxf(gm[i], sc[w][e] + ((corr && !mode) ? corr[e] : 0.f));
          open[w][e] = 0;
        }
    }
    uint32_t used = 0;
    for (int k = 0; k < keep; ++k) {
      float best = -INFINITY;
      int bi = 0x7fffffff;
      for (int i = 0; i < 4; ++i) {
        const int g = lane + 64 * i;
        if (g < groups && !((used >> i) & 1u) && (gm[i] > best || bi == 0x7fffffff)) { best = gm[i]; bi = g; }
      }
      for (int o = 32; o > 0; o >>= 1) {
        const float ob = __shfl_xor(best, o, 64);
        const int oi = __shfl_xor(bi, o, 64);
        if (oi != 0x7fffffff && (bi == 0x7fffffff || ob > best || (ob == best && oi < bi))) { best = ob; bi = oi; }
      }
      if ((bi & 63) == lane) {
        used |= 1u << (bi >> 6);
        for (int e = bi * n; e < (bi + 1) * n; ++e) open[w][e] = 1;
      }
    }
  }
  if (groups > 1) __syncthreads();
  if (!chooses) return;
  float sum = 0.f, my_s = 0.f, top0 = 0.f;
  int my_id = 0;
  uint32_t taken = 0;   // bit i: this lane's expert e = lane + 64 * i is already chosen
  for (int k = 0; k < topk; ++k) {
    float best = -INFINITY;
    int bi = 0x7fffffff;
    for (int i = 0; i < 4; ++i) {
      const int e = lane + 64 * i;
      if (e < E && !((taken >> i) & 1u) && (groups <= 1 || open[w][e])) {
        const float c = sc[w][e] + ((corr && !mode) ? corr[e] : 0.f);
        if (c > best || (c == best && e < bi)) { best = c; bi = e; }
      }
    }
    for (int o = 32; o > 0; o >>= 1) {
      const float ob = __shfl_xor(best, o, 64);
      const int oi = __shfl_xor(bi, o, 64);
      if (ob > best || (ob == best && oi < bi)) { best = ob; bi = oi; }
    }
    if ((bi & 63) == lane) taken |= 1u << (bi >> 6);
    float s = sc[w][bi];
    if (mode) {           // softmax over the chosen logits: the first chosen one is the largest
      if (k == 0) top0 = s;
      s = expf(s - top0);
    }
    sum += s;
    if (lane == k) { my_s = s; my_id = bi; }
  }
  if (live && lane < topk) {
    ids[(long)t * topk + lane] = my_id;
    wts[(long)t * topk + lane] = ((renorm || mode) ? my_s / (sum + 1e-20f) : my_s) * scale;
  }
}

// h[p][f] = silu(Wg[e_p][f] . x[t_p]) * (Wu[e_p][f] . x[t_p]),  p = t * topk + slot; a wave per (p, f).
// clamp: g = min(Wg x, limit), u = clamp(Wu x, -limit, limit), h = g sigmoid(slope g) (u + 1) instead.
// Wg null: no gate, h = max(Wu x, 0)^2.  VEC values of a row per load.
template <typename T, int VEC>
LA_DEV float dot_slice(const T* __restrict__ w, const float (&x)[VEC]) {
  typedef T vec __attribute__((ext_vector_type(VEC)));
  const vec v = *(const vec*)w;
  float a = 0.f;
#pragma unroll
  for (int j = 0; j < VEC; ++j) a = fmaf((float)v[j], x[j], a);
  return a;
}
template <typename T, int VEC>
LA_DEV void row_slice(const T* __restrict__ p, float (&x)[VEC]) {
  typedef T vec __attribute__((ext_vector_type(VEC)));
  const vec v = *(const vec*)p;
#pragma unroll
  for (int j = 0; j < VEC; ++j) x[j] = (float)v[j];
}

template <typename AT, typename WT, int VEC>
__global__ __launch_bounds__(256) void moe_pair_glu_kernel(const AT* __restrict__ x, const WT* __restrict__ wg,
                                                           const WT* __restrict__ wu, const int* __restrict__ ids,
                                                           int topk, int D, int F, int E, AT* __restrict__ h, int clamp,
                                                           float limit, float slope) {
  const int p = blockIdx.y;
  const int f = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (f >= F) return;
  const int e = ids[p];
  if (e < 0 || e >= E) { if (lane == 0) h[(long)p * F + f] = (AT)0.f; return; }
  const AT* xr = x + (long)(p / topk) * D;
  const WT* g = wg ? wg + ((long)e * F + f) * D : nullptr;
  const WT* u = wu + ((long)e * F + f) * D;
  float a = 0.f, b = 0.f;
#pragma unroll 4
  for (int d = lane * VEC; d < D; d += 64 * VEC) {
    float xv[VEC];
    row_slice<AT, VEC>(xr + d, xv);
    if (g) a += dot_slice<WT, VEC>(g + d, xv);
    b += dot_slice<WT, VEC>(u + d, xv);
  }
  a = wave_sum(a);
  b = wave_sum(b);
  if (lane == 0) {
    float v;
    if (!g) {
      const float r = fmaxf(b, 0.f);
      v = r * r;
    } else if (clamp) {
      const float g2 = fminf(a, limit), u2 = fminf(fmaxf(b, -limit), limit);
      v = g2 / (1.f + expf(-slope * g2)) * (u2 + 1.f);
    } else {
      v = silu(a) * b;
    }
    h[(long)p * F + f] = (AT)v;
  }
}

// y[t][d] = sum_slot w[p] * (Wd[e_p][d] . h[p]); a wave per (t, d), slots in order (deterministic)
template <typename AT, typename WT, int VEC>
__global__ __launch_bounds__(256) void moe_pair_down_kernel(const AT* __restrict__ h, const WT* __restrict__ wd,
                                                            const int* __restrict__ ids, const float* __restrict__ wts,
                                                            int topk, int D, int F, int E, float* __restrict__ y) {
  const int t = blockIdx.y;
  const int d = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (d >= D) return;
  float acc = 0.f;
  for (int k = 0; k < topk; ++k) {
    const int p = t * topk + k, e = ids[p];
    if (e < 0 || e >= E) continue;
    const WT* wr = wd + ((long)e * D + d) * F;
    const AT* hr = h + (long)p * F;
    float a = 0.f;
#pragma unroll 4
    for (int f = lane * VEC; f < F; f += 64 * VEC) {
      float hv[VEC];
      row_slice<AT, VEC>(hr + f, hv);
      a += dot_slice<WT, VEC>(wr + f, hv);
    }
    acc = fmaf(wts[p], wave_sum(a), acc);
  }
  if (lane == 0) y[(long)t * D + d] = acc;
}

}  // namespace la

extern "C" int la_router_topk(int f32, int mode, const void* x, long ldx, const void* router, const void* corr, int E,
                              int D, int T, int topk, int renorm, int groups, int keep, float scale, void* ids,
                              void* wts, void* stream) {
  using namespace la;
  if (E < 1 || E > 256 || topk < 1 || topk > E || topk > 64 || T <= 0 || mode < 0 || mode > 1) return -1;
  if (groups < 1 || E % groups || (groups > 1 && (keep < 1 || keep > groups || topk > keep * (E / groups)))) return -2;
  const bool spread = T <= 512;
  const int nw = E > 32 ? 16 : (E + 1) / 2;
#define LA_RT(AT, SP)                                                                                                   \
  hipLaunchKernelGGL((router_topk_kernel<AT, SP>), dim3(SP ? T : (T + 3) / 4), dim3(SP ? 64 * nw : 256), 0,             \
                     (hipStream_t)stream, (const AT*)x, ldx, (const float*)router, (const float*)corr, E, D, T, topk,   \
                     renorm, mode, groups, keep, scale, (int*)ids, (float*)wts)
  if (f32) {
    if (spread) LA_RT(float, true); else LA_RT(float, false);
  } else {
    if (spread) LA_RT(bf16, true); else LA_RT(bf16, false);
  }
#undef LA_RT
  return (int)hipGetLastError();
}

extern "C" int la_router_sigmoid(int f32, const void* x, long ldx, const void* router, const void* corr, int E, int D,
                                 int T, int topk, int renorm, void* ids, void* wts, void* stream) {
  return la_router_topk(f32, 0, x, ldx, router, corr, E, D, T, topk, renorm, 1, 1, 1.f, ids, wts, stream);
}

// f32: activations and weights fp32 (else both bf16).  wg null: ungated experts, relu squared.  x [T, D], wg / wu [E, F, D], wd [E, D, F],
// ids [T * topk], wts [T * topk] -> h [T * topk, F] (scratch, activation type), y [T, D] fp32.
extern "C" int la_moe_pairs(int f32, const void* x, const void* wg, const void* wu, const void* wd, const void* ids,
                            const void* wts, int T, int topk, int D, int F, int E, void* h, void* y, int clamp, float limit,
                            float slope, void* stream) {
  using namespace la;
  if (T <= 0 || topk < 1 || D < 1 || F < 1) return -1;
  const int P = T * topk;
  if (P > 65535 || T > 65535) return -2;
  dim3 g1((F + 3) / 4, P), g2((D + 3) / 4, T);
  hipStream_t s = (hipStream_t)stream;
  if (!x || !wu || !wd || !ids || !wts || !h || !y || (clamp && !wg)) return -3;
#define LA_MP(AT, VEC)                                                                                                    \
  {                                                                                                                       \
    hipLaunchKernelGGL((moe_pair_glu_kernel<AT, AT, VEC>), g1, dim3(256), 0, s, (const AT*)x, (const AT*)wg,              \
                       (const AT*)wu, (const int*)ids, topk, D, F, E, (AT*)h, clamp, limit, slope);                       \
    hipLaunchKernelGGL((moe_pair_down_kernel<AT, AT, VEC>), g2, dim3(256), 0, s, (const AT*)h, (const AT*)wd,             \
                       (const int*)ids, (const float*)wts, topk, D, F, E, (float*)y);                                     \
  }
  // whole vectors of 16 bytes where both widths allow
  const bool al = (((uintptr_t)x | (uintptr_t)wg | (uintptr_t)wu | (uintptr_t)wd | (uintptr_t)h) & 15) == 0;
  if (f32) {
    if (al && !((D | F) & 3)) LA_MP(float, 4) else LA_MP(float, 1)
  } else {
    if (al && !((D | F) & 7)) LA_MP(bf16, 8) else LA_MP(bf16, 1)
  }
#undef LA_MP
  return (int)hipGetLastError();
}
