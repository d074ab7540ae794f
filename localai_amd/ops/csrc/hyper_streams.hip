// Sublayer boundary of a residual kept as n parallel streams (hyper-connections), X [T][n][D] fp32:
//
//   X_to <- sum_from mix[from][to] X_from + outw[to] * (branch + bias)     (all from the old streams)
//   out   = layer norm of u = sum_s inw[s] X_s (inw null: the plain sum), times w plus b
//
// in one launch: the streams' exchange with the finished sublayer's result and the next sublayer's normed
// input.  init (may be null): the streams are not read, every one of them starts as the row init [T][D].
// A workgroup per row.  A thread keeps u of its first KEEP * V columns in registers between the statistics
// and the output; columns beyond that are formed again from the updated streams.  The stream count is a
// runtime number below the template bound SM, so the exchange unrolls with uniform predicates.
#include "row_src.h"

namespace la {

template <int SM, int V, int NT>
__global__ __launch_bounds__(NT) void hyper_streams_kernel(float* __restrict__ X, int n, int D,
                                                           const float* __restrict__ init, RowSrc src, int has_src,
                                                           const float* __restrict__ bias, const float* __restrict__ mix,
                                                           const float* __restrict__ outw, const float* __restrict__ inw,
                                                           const float* __restrict__ w, const float* __restrict__ b,
                                                           float eps, void* __restrict__ out, int out_f32) {
  typedef typename RowVec<V>::type fvec;
  constexpr int KEEP = NT >= 1024 ? 1 : 4;
  __shared__ float red[NT / 64];
  // the exchange's numbers: scalar registers hold those of few streams, LDS those of many
  constexpr bool LC = SM > 4;
  __shared__ float coef[LC ? SM * SM + SM : 1];
  const int t = blockIdx.x, tid = threadIdx.x;
  if constexpr (LC) {
    if (has_src) {
      for (int e = tid; e < n * n + n; e += NT) coef[e] = e < n * n ? mix[e] : outw[e - n * n];
      __syncthreads();
    }
  }
  const long base = (long)t * D;
  float* xr = X + base * n;
  // the updated streams at column c, and u
  auto column = [&](int c) -> fvec {
    fvec x[SM], u = fvec(0.f);
#pragma unroll
    for (int s = 0; s < SM; ++s)
      if (s < n) x[s] = init ? *(const fvec*)(init + base + c) : *(const fvec*)(xr + (long)s * D + c);
    if (!has_src) {
#pragma unroll
      for (int s = 0; s < SM; ++s)
        if (s < n) {
          if (init) *(fvec*)(xr + (long)s * D + c) = x[s];
          const float a = inw ? inw[s] : 1.f;
#pragma unroll
          for (int j = 0; j < V; ++j) u[j] = fmaf(a, x[s][j], u[j]);
        }
      return u;
    }
    fvec y = srcv_at<V>(src, base + c);
    if (bias) {
      const fvec bv = *(const fvec*)(bias + c);
#pragma unroll
      for (int j = 0; j < V; ++j) y[j] += bv[j];
    }
#pragma unroll
    for (int to = 0; to < SM; ++to)
      if (to < n) {
        const float o = LC ? coef[n * n + to] : outw[to], a = inw ? inw[to] : 1.f;
        fvec z;
#pragma unroll
        for (int j = 0; j < V; ++j) z[j] = o * y[j];
#pragma unroll
        for (int s = 0; s < SM; ++s)
          if (s < n) {
            const float m = LC ? coef[s * n + to] : mix[s * n + to];
#pragma unroll
            for (int j = 0; j < V; ++j) z[j] = fmaf(m, x[s][j], z[j]);
          }
        *(fvec*)(xr + (long)to * D + c) = z;
#pragma unroll
        for (int j = 0; j < V; ++j) u[j] = fmaf(a, z[j], u[j]);
      }
    return u;
  };
  // u again, from the streams this thread has already written
  auto again = [&](int c) -> fvec {
    fvec u = fvec(0.f);
    for (int s = 0; s < n; ++s) {
      const fvec x = *(const fvec*)(xr + (long)s * D + c);
      const float a = inw ? inw[s] : 1.f;
#pragma unroll
      for (int j = 0; j < V; ++j) u[j] = fmaf(a, x[j], u[j]);
    }
    return u;
  };
  fvec held[KEEP];
  float sm = 0.f;
  auto add = [&](const fvec& u) {
#pragma unroll
    for (int j = 0; j < V; ++j) sm += u[j];
  };
#pragma unroll
  for (int k = 0; k < KEEP; ++k) {
    const int c = (tid + k * NT) * V;
    if (c < D) {
      held[k] = column(c);
      add(held[k]);
    }
  }
  for (int c = (tid + KEEP * NT) * V; c < D; c += NT * V) add(column(c));
  if (!out) return;                       // uniform: only the streams are asked for
  const float mean = block_sum<NT>(sm, red) / (float)D;
  float ss = 0.f;
  auto sq = [&](const fvec& u) {
#pragma unroll
    for (int j = 0; j < V; ++j) ss = fmaf(u[j] - mean, u[j] - mean, ss);
  };
#pragma unroll
  for (int k = 0; k < KEEP; ++k)
    if ((tid + k * NT) * V < D) sq(held[k]);
  for (int c = (tid + KEEP * NT) * V; c < D; c += NT * V) sq(again(c));
  const float inv = 1.f / sqrtf(block_sum<NT>(ss, red) / (float)D + eps);
  auto emit = [&](int c, const fvec& u) {
    const fvec wv = *(const fvec*)(w + c), bv = *(const fvec*)(b + c);
    fvec o;
#pragma unroll
    for (int j = 0; j < V; ++j) o[j] = fmaf((u[j] - mean) * inv, wv[j], bv[j]);
    putv<V>(out, out_f32, base + c, o);
  };
#pragma unroll
  for (int k = 0; k < KEEP; ++k) {
    const int c = (tid + k * NT) * V;
    if (c < D) emit(c, held[k]);
  }
  for (int c = (tid + KEEP * NT) * V; c < D; c += NT * V) emit(c, again(c));
}

}  // namespace la

extern "C" int la_hyper_streams(void* X, int T, int n, int D, const void* init, const void* sp, int src_f32, long slab, int S,
                                const void* bias, const void* mix, const void* outw, const void* inw, const void* w,
                                const void* b, float eps, void* out, int out_f32, void* stream) {
  using namespace la;
  if (T <= 0 || D <= 0 || n < 1 || n > 16 || !X) return -1;
  if (sp && (!mix || !outw || (src_f32 && S < 1))) return -2;
  if (out && (!w || !b)) return -3;
  RowSrc s{sp, src_f32, slab, S};
  hipStream_t st = (hipStream_t)stream;
#define LA_HS(SM, V, NT)                                                                                                  \
  hipLaunchKernelGGL((hyper_streams_kernel<SM, V, NT>), dim3(T), dim3(NT), 0, st, (float*)X, n, D, (const float*)init, s, \
                     sp != nullptr, (const float*)bias, (const float*)mix, (const float*)outw, (const float*)inw,         \
                     (const float*)w, (const float*)b, eps, out, out_f32)
#define LA_HSN(V, NT)               \
  do {                              \
    if (n <= 2) LA_HS(2, V, NT);    \
    else if (n <= 4) LA_HS(4, V, NT); \
    else LA_HS(16, V, NT);          \
  } while (0)
  if (D & 3) LA_HSN(1, 256);
  else if (T <= 512 && D > 1024) LA_HSN(4, 1024);   // few rows: a row's chain of load latencies is what a launch costs
  else LA_HSN(4, 256);
#undef LA_HSN
#undef LA_HS
  return (int)hipGetLastError();
}
