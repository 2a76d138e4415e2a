// One-element and four-element access of the two projection types (bf16, and fp32 for the engine
// that computes everything in 32-bit), shared by the kernels that are templates over the type.
#pragma once
#include "common.h"

LSA_DEVICE float ld1(const float* p) { return *p; }
LSA_DEVICE float ld1(const bf16_raw* p) { return bf2f(*p); }
LSA_DEVICE void st1(float* p, float v) { *p = v; }
LSA_DEVICE void st1(bf16_raw* p, float v) { *p = f2bf(v); }
LSA_DEVICE void st4(float* p, f32x4_t v) { *reinterpret_cast<f32x4_t*>(p) = v; }
LSA_DEVICE void st4(bf16_raw* p, f32x4_t v) {
  const unsigned lo = (unsigned)f2bf(v[0]) | ((unsigned)f2bf(v[1]) << 16);
  const unsigned hi = (unsigned)f2bf(v[2]) | ((unsigned)f2bf(v[3]) << 16);
  *reinterpret_cast<u32x2_t*>(p) = u32x2_t{lo, hi};
}

LSA_DEVICE float sigmoid(float z) { return 1.0f / (1.0f + __expf(-z)); }
