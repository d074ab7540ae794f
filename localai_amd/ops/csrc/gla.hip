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

// Sum over W lanes (16 or 32 neighbours) of 16 values at once: at every level a lane hands half of its values to its
// partner and keeps the other half, so lane l ends with the total of value l & 15.
template <int W>
LA_DEV float fold16(float (&v)[16], int lane) {
  if constexpr (W == 32) {
#pragma unroll
    for (int j = 0; j < 16; ++j) v[j] += __shfl_xor(v[j], 16, 64);
  }
#pragma unroll
  for (int m = 8; m > 0; m >>= 1) {
    const bool up = lane & m;
#pragma unroll
    for (int j = 0; j < 8; ++j)
      if (j < m) {
        const float keep = up ? v[j + m] : v[j], give = up ? v[j] : v[j + m];
        v[j] = keep + __shfl_xor(give, m, 64);
      }
  }
  return v[0];
}

// qd [chunk][H][16][DkP]: q e^b (times qscale);  kd [chunk][H][DkP][16]: k e^(b_last - b);  dl [chunk][H][DkP]: e^(b_last);
// am [chunk][H][16][16]: A.  DkP = Dk rounded up to 16, filled up with zeros (dl: ones).  Rows past the portion's
// end count as q = k = 0 with decay 1.  A workgroup per (chunk, head); LDS: q, k, b as [16][DkP + 1], then the sums of
// a over the 16 / TPT token ranges of every channel (a thread takes TPT tokens of one channel).
// A in 4 x 4 tiles of (t, s): the four on the diagonal pair by pair (16 lanes each, wave 0), the six below it (32
// lanes each, waves 1 - 3) through the sum b at the tile's first row, c: e^(b_t - b_s) = e^(b_t - c) e^(c - b_s), neither above 1.
template <typename AT, int TPT>
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
  float* tot = bs + GL_C * W;            // [16 / TPT][DkP]
  const int seq = blockIdx.x / maxchunk, c = blockIdx.x - seq * maxchunk, h = blockIdx.y, tid = threadIdx.x;
  const int a0 = cu_q[seq], a = a0 + c * GL_C, n = min(GL_C, cu_q[seq + 1] - a);
  if (n <= 0) return;
  const long no = chunk_no(a0, seq, c) * H + h;
  constexpr int SP = GL_C / TPT;
  const int d = tid % DkP, part = tid / DkP, t0 = part * TPT;
  const bool mine = part < SP, in = mine && d < Dk;     // DkP SP <= GL_NT
  float q[TPT], k[TPT], b[TPT], run = 0.f;
  if (mine) {
#pragma unroll
    for (int i = 0; i < TPT; ++i) {
      const int t = t0 + i;
      const long r = (long)(a + min(t, n - 1));           // rows past the end: loaded, not used
      const int dd = min(d, Dk - 1);
      q[i] = (float)src[r * ld + (long)h * Dk + dd];
      k[i] = (float)src[r * ld + (long)(H + h) * Dk + dd];
      b[i] = (float)z[r * H * Dk + (long)h * Dk + dd];
    }
    const float zbv = in ? zb[h * Dk + d] : 0.f;
#pragma unroll
    for (int i = 0; i < TPT; ++i) {
      const bool live = in && t0 + i < n;
      q[i] = live ? q[i] * qscale : 0.f;
      k[i] = live ? k[i] : 0.f;
      if (live) run += gl_log_decay(b[i] + zbv, inv_tau);
      b[i] = run;
    }
    tot[part * DkP + d] = run;
  }
  __syncthreads();
  if (mine) {
    float before = 0.f, last = 0.f;
#pragma unroll
    for (int s = 0; s < SP; ++s) {
      const float x = tot[s * DkP + d];
      if (s < part) before += x;
      last += x;
    }
#pragma unroll
    for (int i = 0; i < TPT; ++i) {
      const int t = t0 + i;
      b[i] += before;
      qs[t * W + d] = q[i];
      ks[t * W + d] = k[i];
      bs[t * W + d] = b[i];
      qd[(no * GL_C + t) * DkP + d] = q[i] * exp2f(b[i]);
    }
#pragma unroll
    for (int i = 0; i < TPT; i += 4) {
      f32x4 y;
#pragma unroll
      for (int j = 0; j < 4; ++j) y[j] = k[i + j] * exp2f(fminf(last - b[i + j], 0.f));
      *(f32x4*)(kd + (no * DkP + d) * GL_C + t0 + i) = y;
    }
    if (part == 0) dl[no * DkP + d] = exp2f(last);
  }
  __syncthreads();
  float* ar = am + no * GL_C * GL_C;
  const int lane = tid & 63, wave = tid >> 6;
  float acc[16];
#pragma unroll
  for (int e = 0; e < 16; ++e) acc[e] = 0.f;
  if (wave == 0) {
    const int T4 = (lane >> 4) * 4;
    for (int x = lane & 15; x < DkP; x += 16) {
      float qv[4], kv[4], bv[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        qv[i] = qs[(T4 + i) * W + x];
        kv[i] = ks[(T4 + i) * W + x];
        bv[i] = bs[(T4 + i) * W + x];
      }
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j <= i; ++j) acc[4 * i + j] = fmaf(qv[i] * kv[j], i == j ? 1.f : exp2f(bv[i] - bv[j]), acc[4 * i + j]);
    }
    const float v = fold16<16>(acc, lane);
    ar[(T4 + ((lane & 15) >> 2)) * GL_C + T4 + (lane & 3)] = v;
  } else {
    const int u = 2 * (wave - 1) + (lane >> 5);           // tiles (1,0) (2,0) (2,1) (3,0) (3,1) (3,2)
    const int I = u == 0 ? 1 : (u < 3 ? 2 : 3), J = u - I * (I - 1) / 2;
    for (int x = lane & 31; x < DkP; x += 32) {
      const float cb = bs[4 * I * W + x];
      float qv[4], kv[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        qv[i] = qs[(4 * I + i) * W + x] * exp2f(bs[(4 * I + i) * W + x] - cb);
        kv[i] = ks[(4 * J + i) * W + x] * exp2f(cb - bs[(4 * J + i) * W + x]);
      }
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[4 * i + j] = fmaf(qv[i], kv[j], acc[4 * i + j]);
    }
    const float v = fold16<32>(acc, lane);
    const int i = (lane & 15) >> 2, j = lane & 3;
    if (lane & 16) ar[(4 * J + j) * GL_C + 4 * I + i] = 0.f;      // its mirror above the diagonal
    else ar[(4 * I + i) * GL_C + 4 * J + j] = v;
  }
}

// grid (H, nseq, column groups), blockDim / 64 waves: one (portion, head, 16 value columns) per wave
template <typename AT, int KB>
__global__ __launch_bounds__(GL_NT) __attribute__((amdgpu_waves_per_eu(1))) void gla_scan_kernel(const AT* __restrict__ src, long ld, int H, int Dk, int Dv,
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
  // v of rows past the portion's end and of columns past Dv is some other element: their k and A are 0, their column is
  // not stored.  No load behind a branch, so that a chunk's operands fly during the chunk before.
  const AT* vp = src + 2L * H * Dk + (long)h * Dv + min(col, Dv - 1);
  const int nch = (b - a + GL_C - 1) / GL_C;
  struct Ops {
    f32x4 q[KB], k[KB], d[KB], a;
    AT v[4];
  };
  auto load = [&](int c, Ops& x) {
    const long no = chunk_no(a, seq, c) * H + h;
    const float* qp = qd + (no * GL_C + r) * DkP + 4 * g;
    const float* kp = kd + (no * DkP + r) * GL_C + 4 * g;
    const float* dp = dl + no * DkP + 4 * g;
#pragma unroll
    for (int i = 0; i < 4; ++i) x.v[i] = vp[(long)min(a + c * GL_C + 4 * g + i, b - 1) * ld];
    x.a = *(const f32x4*)(am + (no * GL_C + r) * GL_C + 4 * g);
#pragma unroll
    for (int kb = 0; kb < KB; ++kb) {
      x.q[kb] = *(const f32x4*)(qp + 16 * kb);
      x.d[kb] = *(const f32x4*)(dp + 16 * kb);
      x.k[kb] = *(const f32x4*)(kp + 16 * kb * GL_C);
    }
  };
  auto step = [&](int c, const Ops& x) {
    f32x4 oc[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};   // two chains of the read-out's sum
    float vf[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      vf[i] = (float)x.v[i];
      oc[i & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.a[i], vf[i], oc[i & 1], 0, 0, 0);
    }
#pragma unroll
    for (int kb = 0; kb < KB; ++kb) {
#pragma unroll
      for (int i = 0; i < 4; ++i) oc[i & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.q[kb][i], S[kb][i], oc[i & 1], 0, 0, 0);
#pragma unroll
      for (int i = 0; i < 4; ++i) S[kb][i] *= x.d[kb][i];
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int kb = 0; kb < KB; ++kb) S[kb] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.k[kb][i], vf[i], S[kb], 0, 0, 0);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = a + c * GL_C + 4 * g + i;
      if (mine && t < b) o[((long)t * H + h) * Dv + col] = oc[0][i] + oc[1][i];
    }
  };
  Ops x0, x1;
  load(0, x0);
  for (int c = 0; c < nch; c += 2) {
    load(min(c + 1, nch - 1), x1);
    __builtin_amdgcn_sched_barrier(0);     // the loads stay ahead of the chunk they fly over
    step(c, x0);
    __builtin_amdgcn_sched_barrier(0);
    if (c + 1 >= nch) break;
    load(min(c + 2, nch - 1), x0);
    __builtin_amdgcn_sched_barrier(0);
    step(c + 1, x1);
    __builtin_amdgcn_sched_barrier(0);
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
  const int sp = DkP <= 64 ? 4 : (DkP <= 128 ? 2 : 1);      // threads a channel
  const size_t shm = (size_t)(3 * GL_C * (DkP + 1) + sp * DkP) * sizeof(float);
#define LA_GLK(TPT)                                                                                                      \
  {                                                                                                                      \
    if (shm > 48 * 1024)                                                                                                 \
      (void)hipFuncSetAttribute((const void*)gla_chunk_kernel<AT, TPT>, hipFuncAttributeMaxDynamicSharedMemorySize,      \
                                (int)shm);                                                                               \
    hipLaunchKernelGGL((gla_chunk_kernel<AT, TPT>), dim3(nseq * maxchunk, H), dim3(GL_NT), shm, st, src, ld, z, zb,      \
                       inv_tau, H, Dk, DkP, cu_q, maxchunk, qscale, qd, kd, dl, am);                                     \
  }
  if (sp == 4) LA_GLK(4) else if (sp == 2) LA_GLK(8) else LA_GLK(16)
#undef LA_GLK
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
