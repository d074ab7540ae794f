// Rows of a GEMM result as the framework hands them on (fp32 split-K slabs [S][T][N], summed where they are
// read, or one bf16 / fp32 matrix), and stores in the output type.
#pragma once
#include "common.h"

namespace la {

struct RowSrc {
  const void* p;
  int f32;
  long slab;
  int S;
};

LA_DEV float src_at(const RowSrc& s, long idx) {
  if (s.f32) {
    const float* f = (const float*)s.p;
    float a = f[idx];
    for (int k = 1; k < s.S; ++k) a += f[idx + k * s.slab];
    return a;
  }
  return (float)((const bf16*)s.p)[idx];
}

// four neighbouring columns; slabs are requested four at a time (clamped index, masked: no branch between loads)
LA_DEV f32x4 src4_at(const RowSrc& s, long idx) {
  if (!s.f32) {
    const bf16x4 b = *(const bf16x4*)((const bf16*)s.p + idx);
    return f32x4{(float)b[0], (float)b[1], (float)b[2], (float)b[3]};
  }
  const float* f = (const float*)s.p + idx;
  if (s.S <= 1) return *(const f32x4*)f;
  f32x4 a = {0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < s.S; k0 += 4) {
    f32x4 t[4];
#pragma unroll
    for (int k = 0; k < 4; ++k) t[k] = *(const f32x4*)(f + (long)min(k0 + k, s.S - 1) * s.slab);
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const float m = k0 + k < s.S ? 1.f : 0.f;
#pragma unroll
      for (int j = 0; j < 4; ++j) a[j] = fmaf(m, t[k][j], a[j]);
    }
  }
  return a;
}

LA_DEV void put4(void* out, int out_f32, long idx, const f32x4& v) {
  if (out_f32) *(f32x4*)((float*)out + idx) = v;
  else *(bf16x4*)((bf16*)out + idx) = bf16x4{(bf16)v[0], (bf16)v[1], (bf16)v[2], (bf16)v[3]};
}

LA_DEV void put(void* out, int out_f32, long idx, float v) {
  if (out_f32) ((float*)out)[idx] = v;
  else ((bf16*)out)[idx] = (bf16)v;
}

// V neighbouring columns of a row (V = 4: vector accesses; V = 1: any column)
template <int V>
struct RowVec {
  typedef float type __attribute__((ext_vector_type(V)));
};
template <int V>
LA_DEV typename RowVec<V>::type srcv_at(const RowSrc& s, long idx) {
  static_assert(V == 1 || V == 4, "one or four columns");
  if constexpr (V == 4) return src4_at(s, idx);
  else return typename RowVec<V>::type(src_at(s, idx));
}
template <int V>
LA_DEV void putv(void* out, int out_f32, long idx, const typename RowVec<V>::type& v) {
  if constexpr (V == 4) put4(out, out_f32, idx, v);
  else put(out, out_f32, idx, v[0]);
}

}  // namespace la
