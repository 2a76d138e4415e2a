// What the kernels that work on rows of an fp32 stream share (stream_ops.hip, stream_mix.hip).
#pragma once
#include "elem.h"

template <typename T>
LSA_DEVICE f32x4_t load4(const T* p) {
  if constexpr (sizeof(T) == 4) {
    return *reinterpret_cast<const f32x4_t*>(p);
  } else {
    const u32x2_t v = *reinterpret_cast<const u32x2_t*>(p);
    return f32x4_t{__uint_as_float(v[0] << 16), __uint_as_float(v[0] & 0xffff0000u), __uint_as_float(v[1] << 16),
                   __uint_as_float(v[1] & 0xffff0000u)};
  }
}

// V (4 or 1) values
template <int V, typename P>
LSA_DEVICE void get(const P* p, float* f) {
  if constexpr (V == 4) {
    const f32x4_t v = load4(p);
#pragma unroll
    for (int k = 0; k < 4; ++k) f[k] = v[k];
  } else {
    f[0] = ld1(p);
  }
}

// y += the weighted sum of a row's expert results (moe.h) at columns c .. c + V
template <int V, typename T>
LSA_DEVICE void add_pairs(const T* ye, int ldye, const float* weight, const int* place, int top, int row, int c, float* y) {
  for (int e0 = 0; e0 < top; e0 += 4) {  // four results requested at a time
    float z[4][V], w[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int i = row * top + min(e0 + e, top - 1);
      w[e] = e0 + e < top ? weight[i] : 0.f;
      get<V>(ye + (size_t)place[i] * ldye + c, z[e]);
    }
#pragma unroll
    for (int e = 0; e < 4; ++e)
#pragma unroll
      for (int k = 0; k < V; ++k) y[k] = fmaf(w[e], z[e][k], y[k]);
  }
}

// sum over the NT threads of a workgroup
template <int NT>
LSA_DEVICE float row_sum(float s, float* s_part) {
  s = wave_sum(s);
  __syncthreads();  // the sum before this one has been read
  if ((threadIdx.x & 63) == 0) s_part[threadIdx.x >> 6] = s;
  __syncthreads();
  float sum = 0.f;
#pragma unroll
  for (int i = 0; i < NT / 64; ++i) sum += s_part[i];
  return sum;
}
