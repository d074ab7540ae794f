// Gated linear attention: one decay per head and key channel, no softmax and no denominator.
//
//   a_(t,d) = log sigmoid(z_(t,d) + bias_d) / tau        (the decay's logarithm, <= 0)
//   S_t = diag(e^(a_t)) S_(t-1) + k_t v_t^T   (Dk x Dv per head, fp32);   o_t = qscale S_t^T q_t
//   out_t = o_t / sqrt(mean_d o_t[d]^2 + eps) * w_d * silu(gate_t)         (mean over the head's Dv)
//
// The state of a sequence lives in a slot pool [slots][H][Dv][Dk] (value-column major) between launches: a
// portion that starts at position 0 starts from zeros whatever the slot holds, any other from the slot, and
// every portion leaves its end state there.
//
// Batches of one row per sequence (decoding): gla_step_kernel, a workgroup per (sequence, head).  Its state is
// streamed through once, P lanes on a value column's Dk contiguous entries (their decays, k and q stay in
// registers over all columns), and the head's norm and gate are applied before the row leaves.
//
// Portions: chunks of GL_C = 16 tokens, counted from the portion's start.  With b_t the running sum of a
// within the chunk (b_last its end), everything is a product of e^(non-positive), whatever the decays:
//   o_t   = (q_t e^(b_t))^T S_start + sum_(s <= t) A_ts v_s,   A_ts = sum_d q_td k_sd e^(b_td - b_sd)
//   S_end = diag(e^(b_last)) S_start + sum_s (k_s e^(b_last - b_s)) v_s^T
// gla_chunk_kernel forms the operands of every chunk, all chunks of the batch in parallel.  gla_scan_kernel
// walks the chunks of one (portion, head, 16 value columns) with one wave on the fp32 matrix instructions:
// the wave's state columns stay in accumulators, laid out (row 4 g + i, column lane & 15, g = lane >> 4) such that
// register i of 16 state rows is itself a right operand (4 rows: i, 4 + i, 8 + i, 12 + i) of q S; left operands
// are stored so that each lane reads its 4 values of 16 as one vector.  gla_out_kernel: norm and gate.
#include "common.h"

namespace la {

constexpr int GL_NT = 256;
constexpr int GL_C = 16;
constexpr float GL_LOG2E = 1.4426950408889634f;

// log2 of sigmoid(x)^(1 / tau), inv_tau = log2(e) / tau
LA_DEV float gl_log_decay(float x, float inv_tau) { return -(fmaxf(-x, 0.f) + log1pf(expf(-fabsf(x)))) * inv_tau; }

// ---------------------------------------------------------------------------------------- decoding
template <typename AT, int V, int R>
__global__ __launch_bounds__(GL_NT) void gla_step_kernel(const AT* __restrict__ src, long ld, long gcol,
                                                         const AT* __restrict__ z, const float* __restrict__ zb,
                                                         float inv_tau, int H, int Dk, int Dv, int P,
                                                         const int* __restrict__ pos, const int* __restrict__ sslots,
                                                         float* __restrict__ state, float qscale,
                                                         const float* __restrict__ w, float eps, AT* __restrict__ out) {
  typedef float fvec __attribute__((ext_vector_type(V)));
  extern __shared__ float os[];            // [Dv] the head's read-out
  __shared__ float red[GL_NT / 64];
  const int h = blockIdx.x, t = blockIdx.y, tid = threadIdx.x;
  const int part = tid % P, grp = tid / P, ng = GL_NT / P;
  const AT* row = src + (long)t * ld;
  const AT* q = row + (long)h * Dk;
  const AT* k = row + (long)(H + h) * Dk;
  const AT* v = row + 2L * H * Dk + (long)h * Dv;
  const int slot = sslots[t];
  float* st = slot >= 0 ? state + ((long)slot * H + h) * Dv * Dk : nullptr;
  const bool zero = !st || pos[t] == 0;
  float a[R][V], kk[R][V], qq[R][V];
#pragma unroll
  for (int r = 0; r < R; ++r)
#pragma unroll
    for (int j = 0; j < V; ++j) {
      const int d = (r * P + part) * V + j;
      const bool in = d < Dk;
      a[r][j] = in ? exp2f(gl_log_decay((float)z[(long)t * H * Dk + (long)h * Dk + d] + zb[h * Dk + d], inv_tau)) : 0.f;
      kk[r][j] = in ? (float)k[d] : 0.f;
      qq[r][j] = in ? (float)q[d] * qscale : 0.f;
    }
  constexpr int UN = 4;                    // columns a lane group has in flight
  for (int c0 = grp; c0 < Dv; c0 += ng * UN) {
    fvec s[UN][R];
#pragma unroll
    for (int u = 0; u < UN; ++u)
#pragma unroll
      for (int r = 0; r < R; ++r) {
        const int c = c0 + u * ng, d = (r * P + part) * V;
        s[u][r] = fvec(0.f);
        if (!zero && c < Dv && d < Dk) s[u][r] = *(const fvec*)(st + (long)c * Dk + d);
      }
#pragma unroll
    for (int u = 0; u < UN; ++u) {
      const int c = c0 + u * ng;
      const float vc = c < Dv ? (float)v[c] : 0.f;
      float o = 0.f;
#pragma unroll
      for (int r = 0; r < R; ++r) {
        const int d = (r * P + part) * V;
#pragma unroll
        for (int j = 0; j < V; ++j) {
          s[u][r][j] = fmaf(a[r][j], s[u][r][j], kk[r][j] * vc);
          o = fmaf(s[u][r][j], qq[r][j], o);
        }
        if (st && c < Dv && d < Dk) *(fvec*)(st + (long)c * Dk + d) = s[u][r];
      }
      for (int x = P >> 1; x > 0; x >>= 1) o += __shfl_xor(o, x, 64);
      if (part == 0 && c < Dv) os[c] = o;
    }
  }
  __syncthreads();
  float ss = 0.f;
  for (int c = tid; c < Dv; c += GL_NT) ss = fmaf(os[c], os[c], ss);
  const float inv = 1.f / sqrtf(block_sum<GL_NT>(ss, red) / (float)Dv + eps);
  const AT* g = row + gcol + (long)h * Dv;
  for (int c = tid; c < Dv; c += GL_NT) {
    const float gv = (float)g[c];
    out[((long)t * H + h) * Dv + c] = (AT)(os[c] * inv * w[c] * (gv / (1.f + expf(-gv))));
  }
}

// ---------------------------------------------------------------------------------------- portions
// Chunk c of the portion of sequence seq that starts at row a has the number a / 16 + seq + c (unique, below T / 16 + nseq).
LA_DEV long chunk_no(int a, int seq, int c) { return a / GL_C + seq + c; }

// qd [chunk][H][16][DkP]: q e^b (times qscale);  kd [chunk][H][DkP][16]: k e^(b_last - b);  dl [chunk][H][DkP]: e^(b_last);
// am [chunk][H][16][16]: A.  DkP = Dk rounded up to 16, filled up with zeros (dl: ones).  Rows past the portion's
// end count as q = k = 0 with decay 1.  A workgroup per (chunk, head); LDS: q, k, b as [16][DkP + 1].
template <typename AT>
__global__ __launch_bounds__(GL_NT) void gla_chunk_kernel(const AT* __restrict__ src, long ld, const AT* __restrict__ z,
                                                          const float* __restrict__ zb, float inv_tau, int H, int Dk,
                                                          int DkP, const int* __restrict__ cu_q, int maxchunk, float qscale,
                                                          float* __restrict__ qd, float* __restrict__ kd,
                                                          float* __restrict__ dl, float* __restrict__ am) {
  extern __shared__ float lds[];
  const int W = DkP + 1;
  float* qs = lds;
  float* ks = qs + GL_C * W;
  float* bs = ks + GL_C * W;
  const int seq = blockIdx.x / maxchunk, c = blockIdx.x - seq * maxchunk, h = blockIdx.y, tid = threadIdx.x;
  const int a0 = cu_q[seq], a = a0 + c * GL_C, n = min(GL_C, cu_q[seq + 1] - a);
  if (n <= 0) return;
  const long no = chunk_no(a0, seq, c) * H + h;
  for (int d = tid; d < DkP; d += GL_NT) {
    const bool in = d < Dk;
    const float zbv = in ? zb[h * Dk + d] : 0.f;
    float q[GL_C], k[GL_C], b[GL_C], run = 0.f;
#pragma unroll
    for (int t = 0; t < GL_C; ++t) {
      const bool live = in && t < n;
      const long r = (long)(a + (t < n ? t : 0));
      q[t] = live ? (float)src[r * ld + (long)h * Dk + d] * qscale : 0.f;
      k[t] = live ? (float)src[r * ld + (long)(H + h) * Dk + d] : 0.f;
      b[t] = live ? (float)z[r * H * Dk + (long)h * Dk + d] : 0.f;
    }
#pragma unroll
    for (int t = 0; t < GL_C; ++t) {
      if (in && t < n) run += gl_log_decay(b[t] + zbv, inv_tau);
      b[t] = run;
      qs[t * W + d] = q[t];
      ks[t * W + d] = k[t];
      bs[t * W + d] = run;
      qd[(no * GL_C + t) * DkP + d] = q[t] * exp2f(run);
    }
#pragma unroll
    for (int t = 0; t < GL_C; t += 4) {
      f32x4 y;
#pragma unroll
      for (int j = 0; j < 4; ++j) y[j] = k[t + j] * exp2f(run - b[t + j]);
      *(f32x4*)(kd + (no * DkP + d) * GL_C + t) = y;
    }
    dl[no * DkP + d] = exp2f(run);
  }
  __syncthreads();
  // A below and on the diagonal: 136 (t, s) pairs, 8 lanes each; above it zeros
  float* ar = am + no * GL_C * GL_C;
  constexpr int NP = GL_C * (GL_C + 1) / 2, ROUNDS = (NP * 8 + GL_NT - 1) / GL_NT;
  for (int e = tid; e < GL_C * GL_C; e += GL_NT)
    if ((e & (GL_C - 1)) > e / GL_C) ar[e] = 0.f;
#pragma unroll
  for (int i = 0; i < ROUNDS; ++i) {
    const int e = i * GL_NT + tid, p = min(e >> 3, NP - 1), part = e & 7;
    int t = (int)((sqrtf(8.f * p + 1.f) - 1.f) * 0.5f);     // p = t (t + 1) / 2 + s
    if ((t + 1) * (t + 2) / 2 <= p) ++t;
    if (t * (t + 1) / 2 > p) --t;
    const int s = p - t * (t + 1) / 2;
    const float* qr = qs + t * W;
    const float* kr = ks + s * W;
    const float* bt = bs + t * W;
    const float* bq = bs + s * W;
    float acc = 0.f;
    for (int d = part; d < DkP; d += 8) acc = fmaf(qr[d] * kr[d], exp2f(bt[d] - bq[d]), acc);
    acc = group_sum<8>(acc);
    if (part == 0 && (e >> 3) < NP) ar[t * GL_C + s] = acc;
  }
}

// grid (H, nseq, column groups), blockDim / 64 waves: one (portion, head, 16 value columns) per wave
template <typename AT, int KB>
__global__ __launch_bounds__(GL_NT) void gla_scan_kernel(const AT* __restrict__ src, long ld, int H, int Dk, int Dv,
                                                         const int* __restrict__ pos, const int* __restrict__ cu_q,
                                                         const int* __restrict__ sslots, float* __restrict__ state,
                                                         const float* __restrict__ qd, const float* __restrict__ kd,
                                                         const float* __restrict__ dl, const float* __restrict__ am,
                                                         float* __restrict__ o) {
  constexpr int DkP = KB * 16;
  const int h = blockIdx.x, seq = blockIdx.y, tid = threadIdx.x, lane = tid & 63;
  const int col = (blockIdx.z * (blockDim.x >> 6) + (tid >> 6)) * 16 + (lane & 15), r = lane & 15, g = lane >> 4;
  const int a = cu_q[seq], b = cu_q[seq + 1];
  if (b <= a || col - r >= Dv) return;
  const int slot = sslots[seq];
  const bool mine = col < Dv;
  float* st = slot >= 0 && mine ? state + (((long)slot * H + h) * Dv + col) * Dk : nullptr;
  const bool zero = pos[a] == 0;
  f32x4 S[KB];                           // rows 16 kb + 4 g + i of column col
#pragma unroll
  for (int kb = 0; kb < KB; ++kb)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = 16 * kb + 4 * g + i;
      S[kb][i] = st && !zero && d < Dk ? st[d] : 0.f;
    }
  const AT* vp = src + 2L * H * Dk + (long)h * Dv + col;
  const int nch = (b - a + GL_C - 1) / GL_C;
  f32x4 qf[KB], kf[KB], df[KB], af;
  float vf[4];
  auto load = [&](int c, f32x4 (&Q)[KB], f32x4 (&K)[KB], f32x4 (&D)[KB], f32x4& A, float (&Vv)[4]) {
    const long no = chunk_no(a, seq, c) * H + h;
    const float* qp = qd + (no * GL_C + r) * DkP + 4 * g;
    const float* kp = kd + (no * DkP + r) * GL_C + 4 * g;
    const float* dp = dl + no * DkP + 4 * g;
#pragma unroll
    for (int kb = 0; kb < KB; ++kb) {
      Q[kb] = *(const f32x4*)(qp + 16 * kb);
      K[kb] = *(const f32x4*)(kp + 16 * kb * GL_C);
      D[kb] = *(const f32x4*)(dp + 16 * kb);
    }
    A = *(const f32x4*)(am + (no * GL_C + r) * GL_C + 4 * g);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = a + c * GL_C + 4 * g + i;
      Vv[i] = mine && t < b ? (float)vp[(long)t * ld] : 0.f;
    }
  };
  load(0, qf, kf, df, af, vf);
  for (int c = 0; c < nch; ++c) {
    f32x4 qn[KB], kn[KB], dn[KB], an;
    float vn[4];
    load(min(c + 1, nch - 1), qn, kn, dn, an, vn);   // the next chunk's operands fly during this one
    f32x4 oc[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};   // two chains of the read-out's sum
#pragma unroll
    for (int i = 0; i < 4; ++i) oc[i & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(af[i], vf[i], oc[i & 1], 0, 0, 0);
#pragma unroll
    for (int kb = 0; kb < KB; ++kb) {
#pragma unroll
      for (int i = 0; i < 4; ++i)
        oc[i & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(qf[kb][i], S[kb][i], oc[i & 1], 0, 0, 0);
#pragma unroll
      for (int i = 0; i < 4; ++i) S[kb][i] *= df[kb][i];
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int kb = 0; kb < KB; ++kb) S[kb] = __builtin_amdgcn_mfma_f32_16x16x4f32(kf[kb][i], vf[i], S[kb], 0, 0, 0);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = a + c * GL_C + 4 * g + i;
      if (mine && t < b) o[((long)t * H + h) * Dv + col] = oc[0][i] + oc[1][i];
    }
#pragma unroll
    for (int kb = 0; kb < KB; ++kb) {
      qf[kb] = qn[kb];
      kf[kb] = kn[kb];
      df[kb] = dn[kb];
    }
    af = an;
#pragma unroll
    for (int i = 0; i < 4; ++i) vf[i] = vn[i];
  }
  if (!st) return;
#pragma unroll
  for (int kb = 0; kb < KB; ++kb)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = 16 * kb + 4 * g + i;
      if (d < Dk) st[d] = S[kb][i];
    }
}

// out[t][h][:] = o / sqrt(mean(o^2) + eps) * w * silu(gate): LG lanes per (token, head), V values an access
template <typename AT, int V>
__global__ __launch_bounds__(GL_NT) void gla_out_kernel(const float* __restrict__ o, const AT* __restrict__ src, long ld,
                                                        long gcol, int H, int Dv, long rows, int LG,
                                                        const float* __restrict__ w, float eps, AT* __restrict__ out) {
  typedef float fvec __attribute__((ext_vector_type(V)));
  typedef AT avec __attribute__((ext_vector_type(V)));
  const long r = ((long)blockIdx.x * GL_NT + threadIdx.x) / LG;
  if (r >= rows) return;
  const int lane = threadIdx.x % LG;
  const long t = r / H;
  const int h = (int)(r - t * H);
  const float* orow = o + r * Dv;
  fvec first = fvec(0.f);
  float ss = 0.f;
  for (int d = lane * V; d < Dv; d += LG * V) {
    const fvec x = *(const fvec*)(orow + d);
    if (d == lane * V) first = x;
#pragma unroll
    for (int j = 0; j < V; ++j) ss = fmaf(x[j], x[j], ss);
  }
  for (int x = LG >> 1; x > 0; x >>= 1) ss += __shfl_xor(ss, x, 64);
  const float inv = 1.f / sqrtf(ss / (float)Dv + eps);
  const AT* gr = src + t * ld + gcol + (long)h * Dv;
  for (int d = lane * V; d < Dv; d += LG * V) {
    const fvec x = d == lane * V ? first : *(const fvec*)(orow + d);
    const avec gv = *(const avec*)(gr + d);
    const fvec wv = *(const fvec*)(w + d);
    avec y;
#pragma unroll
    for (int j = 0; j < V; ++j) {
      const float gf = (float)gv[j];
      y[j] = (AT)(x[j] * inv * wv[j] * (gf / (1.f + expf(-gf))));
    }
    *(avec*)(out + r * Dv + d) = y;
  }
}

template <typename AT>
static int gla_launch(const AT* src, long ld, const AT* z, const float* zb, float tau, int T, int nseq, int H, int Dk,
                      int Dv, const int* pos, const int* cu_q, const int* sslots, float* state, const float* w, float eps,
                      int single, int max_rows, float* qd, float* kd, float* dl, float* am, float* o, AT* out,
                      hipStream_t st) {
  const float qscale = 1.f / sqrtf((float)Dk), inv_tau = GL_LOG2E / tau;
  const long gcol = 2L * H * Dk + (long)H * Dv;
  if (single) {
    const int V = Dk & 3 ? 1 : 4, need = (Dk + V - 1) / V;
    int P = 4;
    while (P < 64 && P < need) P <<= 1;
    const int R = (need + P - 1) / P;
#define LA_GLS(V, R)                                                                                                      \
  hipLaunchKernelGGL((gla_step_kernel<AT, V, R>), dim3(H, nseq), dim3(GL_NT), Dv * sizeof(float), st, src, ld, gcol, z, zb, \
                     inv_tau, H, Dk, Dv, P, pos, sslots, state, qscale, w, eps, out)
    if (V == 4) LA_GLS(4, 1);       // Dk <= 256: one vector a lane
    else if (R == 1) LA_GLS(1, 1);
    else LA_GLS(1, 4);
#undef LA_GLS
    return (int)hipGetLastError();
  }
  const int KB = (Dk + 15) / 16, maxchunk = (max_rows + GL_C - 1) / GL_C;
  int kbt = 1;                      // instances: 1 .. 4, then 6, 8, 12, 16 blocks of key channels
  for (int v : {1, 2, 3, 4, 6, 8, 12, 16}) {
    kbt = v;
    if (v >= KB) break;
  }
  const int DkP = kbt * 16;
  const size_t shm = (size_t)3 * GL_C * (DkP + 1) * sizeof(float);
  if (shm > 48 * 1024)
    (void)hipFuncSetAttribute((const void*)gla_chunk_kernel<AT>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)shm);
  hipLaunchKernelGGL(gla_chunk_kernel<AT>, dim3(nseq * maxchunk, H), dim3(GL_NT), shm, st, src, ld, z, zb, inv_tau, H, Dk,
                     DkP, cu_q, maxchunk, qscale, qd, kd, dl, am);
  const int blocks = (Dv + 15) / 16, waves = blocks < 4 ? blocks : 4;
#define LA_GLC(KBT)                                                                                                    \
  if (kbt == KBT)                                                                                                      \
    hipLaunchKernelGGL((gla_scan_kernel<AT, KBT>), dim3(H, nseq, (blocks + waves - 1) / waves), dim3(64 * waves), 0, st, \
                       src, ld, H, Dk, Dv, pos, cu_q, sslots, state, (const float*)qd, (const float*)kd,               \
                       (const float*)dl, (const float*)am, o);
  LA_GLC(1) LA_GLC(2) LA_GLC(3) LA_GLC(4) LA_GLC(6) LA_GLC(8) LA_GLC(12) LA_GLC(16)
#undef LA_GLC
  const long rows = (long)T * H;
  const bool vec = !(Dv & 3) && !(ld & 3) && !(gcol & 3) && !(((uintptr_t)src | (uintptr_t)out) & 15);
  int LG = 4;
  while (LG < 64 && LG * (vec ? 4 : 1) < Dv) LG <<= 1;
  const dim3 grid((unsigned)((rows * LG + GL_NT - 1) / GL_NT));
  if (vec)
    hipLaunchKernelGGL((gla_out_kernel<AT, 4>), grid, dim3(GL_NT), 0, st, (const float*)o, src, ld, gcol, H, Dv, rows, LG, w,
                       eps, out);
  else
    hipLaunchKernelGGL((gla_out_kernel<AT, 1>), grid, dim3(GL_NT), 0, st, (const float*)o, src, ld, gcol, H, Dv, rows, LG, w,
                       eps, out);
  return (int)hipGetLastError();
}

}  // namespace la

// key widths the instances cover; the widths of the scratch operands: DkP of a key width (0: out of reach)
extern "C" int la_gla_width(int Dk) {
  for (int v : {1, 2, 3, 4, 6, 8, 12, 16})
    if (Dk > 0 && v * 16 >= Dk) return v * 16;
  return 0;
}

// src rows [q (H Dk) | k (H Dk) | v (H Dv) | gate (H Dv)], row stride ld; z [T][H Dk] decay logits, zb their bias;
// single: one row per sequence (nseq == T; the scratch operands are not used).  max_rows: the longest portion.
// Scratch (fp32, n = (T / 16 + nseq) H): qd, kd [n][16 DkP], dl [n][DkP], am [n][256], o [T][H Dv].
extern "C" int la_gla(int f32, const void* src, long ld, const void* z, const void* zb, float tau, int T, int nseq, int H,
                      int Dk, int Dv, const void* pos, const void* cu_q, const void* sslots, void* state, int nslots,
                      const void* w, float eps, int single, int max_rows, void* qd, void* kd, void* dl, void* am, void* o,
                      void* out, void* stream) {
  using namespace la;
  if (T <= 0 || nseq <= 0 || H <= 0 || Dk <= 0 || Dv <= 0 || nslots <= 0 || !(tau > 0.f) || ld < 2L * H * (Dk + Dv)) return -1;
  if (!src || !z || !zb || !pos || !sslots || !state || !w || !out || la_gla_width(Dk) == 0 || Dv > 8192) return -2;
  if (single ? T != nseq : (!cu_q || !qd || !kd || !dl || !am || !o || max_rows < 1)) return -3;
  hipStream_t st = (hipStream_t)stream;
  if (f32)
    return gla_launch<float>((const float*)src, ld, (const float*)z, (const float*)zb, tau, T, nseq, H, Dk, Dv,
                             (const int*)pos, (const int*)cu_q, (const int*)sslots, (float*)state, (const float*)w, eps,
                             single, max_rows, (float*)qd, (float*)kd, (float*)dl, (float*)am, (float*)o, (float*)out, st);
  return gla_launch<bf16>((const bf16*)src, ld, (const bf16*)z, (const float*)zb, tau, T, nseq, H, Dk, Dv, (const int*)pos,
                          (const int*)cu_q, (const int*)sslots, (float*)state, (const float*)w, eps, single, max_rows,
                          (float*)qd, (float*)kd, (float*)dl, (float*)am, (float*)o, (bf16*)out, st);
}
