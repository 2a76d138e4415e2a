// Kernels of a decoder whose residual stream is fp32 and whose norms sit on the sublayers' OUTPUTS
// (the sublayers read the stream itself):
//   lsa_stream_embed     x = table[id] * scale in fp32 (or several copies side by side: a decoder with several
//                        streams, stream_mix.hip), plus, where asked for, the copy the projections read
//   lsa_stream_add_norm  x += rms(y) * gain: a sublayer's result, RMS-normed, joins the stream (gain
//                        = norm weight times layer scale, fp32), plus the copy the projections read
//   lsa_stream_norm      rms(x) * gain -> the head projection's input
// and of one whose sublayers read a norm of the stream and join it through a sigmoid gate per element:
//   lsa_stream_join      x += sigmoid(g1) * y1 + sigmoid(g2) * (y2, or the weighted sum of a row's expert
//                        results), then (optionally) rms(x) * gain -> the next sublayers' input
// and of one with norms on both sides of its sublayers:
//   lsa_stream_renorm    v = y + the weighted sum of a row's expert results; x (+)= rms(v) * post (or v as it
//                        is), then (optionally) rms(x) * gain -> the next sublayer's input, or x itself
//   lsa_softcap_rows     logits -> cap tanh(logits / cap)
//   lsa_logits_argmax    argmax keys of fp32 logits (the fp32 engine; the bf16 one fuses this
//                        into the head GEMM)
//   lsa_cast_rows        fp32 rows -> the projections' type (a stage's input stream)
// T is the projections' type (bf16, or fp32 for the fp32 engine). Rows of the copies may be wider
// than the stream (GEMM padding): those columns are left as they are (zero).
#include "stream_row.h"

namespace {

template <typename T>
__global__ __launch_bounds__(256) void stream_embed_kernel(const int* __restrict__ ids, const T* __restrict__ table,
                                                           int ldt, float scale, int W, int copies,
                                                           float* __restrict__ x, int ldx, T* __restrict__ xc, int ldc) {
  const int row = blockIdx.x;
  const T* src = table + (size_t)ids[row] * ldt;
  for (int c = threadIdx.x; c < W; c += 256) {
    const float v = ld1(src + c) * scale;
    for (int s = 0; s < copies; ++s) x[(size_t)row * ldx + (size_t)s * W + c] = v;
    if (xc) st1(xc + (size_t)row * ldc + c, v);
  }
}
// bf16, 8 values per thread and step
__global__ __launch_bounds__(256) void stream_embed8_kernel(const int* __restrict__ ids, const bf16_raw* __restrict__ table,
                                                            int ldt, float scale, int W, int copies,
                                                            float* __restrict__ x, int ldx, bf16_raw* __restrict__ xc, int ldc) {
  const int row = blockIdx.x;
  const bf16_raw* src = table + (size_t)ids[row] * ldt;
  for (int c = threadIdx.x * 8; c < W; c += 2048) {
    float f[8];
    unpack8(ld16(src + c), f);
#pragma unroll
    for (int k = 0; k < 8; ++k) f[k] *= scale;
    for (int s = 0; s < copies; ++s) {
      float* d = x + (size_t)row * ldx + (size_t)s * W + c;
      *reinterpret_cast<f32x4_t*>(d) = f32x4_t{f[0], f[1], f[2], f[3]};
      *reinterpret_cast<f32x4_t*>(d + 4) = f32x4_t{f[4], f[5], f[6], f[7]};
    }
    if (xc) st16(xc + (size_t)row * ldc + c, pack8(f));
  }
}

// x -> its copy xc and, where given, x2 (the engine's own stream buffer)
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void cast_rows_kernel(const float* __restrict__ x, int ldx, int W, T* __restrict__ xc,
                                                        int ldc, float* __restrict__ x2, int ldx2) {
  const int row = blockIdx.x;
  const float* s = x + (size_t)row * ldx;
  if constexpr (VEC) {
    for (int c = threadIdx.x * 4; c < W; c += 1024) {
      const f32x4_t v = *reinterpret_cast<const f32x4_t*>(s + c);
      st4(xc + (size_t)row * ldc + c, v);
      if (x2) *reinterpret_cast<f32x4_t*>(x2 + (size_t)row * ldx2 + c) = v;
    }
  } else {
    for (int c = threadIdx.x; c < W; c += 256) {
      st1(xc + (size_t)row * ldc + c, s[c]);
      if (x2) x2[(size_t)row * ldx2 + c] = s[c];
    }
  }
}

// ADD: x += rms(y) * gain and xc = x; else xc = rms(y) * gain. One workgroup per row; a row of up
// to 256 * 4 * NV values stays in registers (NV > 0), longer ones are read twice.
template <typename T, bool ADD, int NV>
__global__ __launch_bounds__(256) void norm_rows_kernel(const float* __restrict__ y, int ldy,
                                                        const float* __restrict__ gain, float eps, int W,
                                                        float* __restrict__ x, int ldx, T* __restrict__ xc, int ldc) {
  __shared__ float s_part[4];
  const int row = blockIdx.x, tid = threadIdx.x;
  const float* yr = y + (size_t)row * ldy;
  float* xr = ADD ? x + (size_t)row * ldx : nullptr;
  T* cr = xc + (size_t)row * ldc;
  float s = 0.f;
  if constexpr (NV > 0) {  // W % 4 == 0, every pointer 16-B aligned
    f32x4_t v[NV], xv[NV];
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int c = (tid + j * 256) * 4;
      v[j] = c < W ? *reinterpret_cast<const f32x4_t*>(yr + c) : f32x4_t{0.f, 0.f, 0.f, 0.f};
      if (ADD) xv[j] = c < W ? *reinterpret_cast<const f32x4_t*>(xr + c) : f32x4_t{0.f, 0.f, 0.f, 0.f};
    }
#pragma unroll
    for (int j = 0; j < NV; ++j)
#pragma unroll
      for (int k = 0; k < 4; ++k) s += v[j][k] * v[j][k];
    s = wave_sum(s);
    if ((tid & 63) == 0) s_part[tid >> 6] = s;
    __syncthreads();
    const float rs = 1.f / sqrtf((s_part[0] + s_part[1] + s_part[2] + s_part[3]) / (float)W + eps);
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int c = (tid + j * 256) * 4;
      if (c >= W) break;
      const f32x4_t g = *reinterpret_cast<const f32x4_t*>(gain + c);
      f32x4_t o;
#pragma unroll
      for (int k = 0; k < 4; ++k) o[k] = (ADD ? xv[j][k] : 0.f) + v[j][k] * rs * g[k];
      if (ADD) *reinterpret_cast<f32x4_t*>(xr + c) = o;
      st4(cr + c, o);
    }
  } else {
    for (int c = tid; c < W; c += 256) s += yr[c] * yr[c];
    s = wave_sum(s);
    if ((tid & 63) == 0) s_part[tid >> 6] = s;
    __syncthreads();
    const float rs = 1.f / sqrtf((s_part[0] + s_part[1] + s_part[2] + s_part[3]) / (float)W + eps);
    for (int c = tid; c < W; c += 256) {
      const float o = (ADD ? xr[c] : 0.f) + yr[c] * rs * gain[c];
      if (ADD) xr[c] = o;
      st1(cr + c, o);
    }
  }
}

template <typename T, bool ADD>
void launch_norm(const float* y, int ldy, const float* gain, float eps, int rows, int W, float* x, int ldx, T* xc,
                 int ldc, hipStream_t s) {
  const bool vec = W % 4 == 0 && ldy % 4 == 0 && ldc % 4 == 0 && (!ADD || ldx % 4 == 0) &&
                   ((uintptr_t)y | (uintptr_t)gain | (uintptr_t)x | (uintptr_t)xc) % 16 == 0;
  const int nv = vec ? (W + 1023) / 1024 : 0;
#define LSA_N(NV) norm_rows_kernel<T, ADD, NV><<<rows, 256, 0, s>>>(y, ldy, gain, eps, W, x, ldx, xc, ldc)
  if (nv >= 1 && nv <= 2) LSA_N(2);
  else if (nv >= 3 && nv <= 4) LSA_N(4);
  else if (nv >= 5 && nv <= 8) LSA_N(8);
  else LSA_N(0);
#undef LSA_N
}

struct JoinArgs {  // Mirrored by llm_sharding_amd/ops/stream.py::JoinArgs
  const float* y1;       // [rows][ldy1] or null
  const void* g1;        // gate logits of y1 / of the second result, in the projections' type
  const void* g2;
  const float* y2;       // [rows][ldy2] or null
  const void* ye;        // [rows * top][ldye] expert results of the sorted pairs, or null
  const float* weight;   // [rows * top]
  const int* place;      // [rows * top] where a row's pair lies in ye
  const float* gain;     // null: no norm
  int ldy1, ldg1, ldg2, ldy2, ldye, top;
  float eps;
};

// what the results add to x[row][c .. c + V)
template <typename T, int V>
LSA_DEVICE void join_at(const JoinArgs& a, int row, int c, float* x) {
  float y[V], g[V];
  if (a.y1) {
    get<V>(a.y1 + (size_t)row * a.ldy1 + c, y);
    get<V>((const T*)a.g1 + (size_t)row * a.ldg1 + c, g);
#pragma unroll
    for (int k = 0; k < V; ++k) x[k] += sigmoid(g[k]) * y[k];
  }
  if (a.y2 || a.ye) {
    get<V>((const T*)a.g2 + (size_t)row * a.ldg2 + c, g);
    if (a.y2) {
      get<V>(a.y2 + (size_t)row * a.ldy2 + c, y);
    } else {
#pragma unroll
      for (int k = 0; k < V; ++k) y[k] = 0.f;
      add_pairs<V>((const T*)a.ye, a.ldye, a.weight, a.place, a.top, row, c, y);
    }
#pragma unroll
    for (int k = 0; k < V; ++k) x[k] += sigmoid(g[k]) * y[k];
  }
}

// NT threads per row. NV > 0: rows of up to 4 NT NV values in registers, four at a time; 0: any width
template <typename T, int NV, int NT>
__global__ __launch_bounds__(NT) void join_kernel(JoinArgs a, int W, float* __restrict__ x, int ldx, T* __restrict__ xc,
                                                   int ldc) {
  __shared__ float s_part[NT / 64];
  const int row = blockIdx.x, tid = threadIdx.x;
  float* xr = x + (size_t)row * ldx;
  float s = 0.f;
  f32x4_t v[NV > 0 ? NV : 1];
  if constexpr (NV > 0) {
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int c = (tid + j * NT) * 4;
      v[j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
      if (c >= W) continue;
      float f[4];
      const f32x4_t x4 = *reinterpret_cast<const f32x4_t*>(xr + c);
#pragma unroll
      for (int k = 0; k < 4; ++k) f[k] = x4[k];
      join_at<T, 4>(a, row, c, f);
      v[j] = f32x4_t{f[0], f[1], f[2], f[3]};
      *reinterpret_cast<f32x4_t*>(xr + c) = v[j];
#pragma unroll
      for (int k = 0; k < 4; ++k) s += f[k] * f[k];
    }
  } else {
    for (int c = tid; c < W; c += NT) {
      float f = xr[c];
      join_at<T, 1>(a, row, c, &f);
      xr[c] = f;
      s += f * f;
    }
  }
  if (!a.gain) return;
  s = wave_sum(s);
  if ((tid & 63) == 0) s_part[tid >> 6] = s;
  __syncthreads();
  float sum = 0.f;
#pragma unroll
  for (int i = 0; i < NT / 64; ++i) sum += s_part[i];
  const float rs = 1.f / sqrtf(sum / (float)W + a.eps);
  T* cr = xc + (size_t)row * ldc;
  if constexpr (NV > 0) {
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int c = (tid + j * NT) * 4;
      if (c < W) st4(cr + c, v[j] * rs * *reinterpret_cast<const f32x4_t*>(a.gain + c));
    }
  } else {
    for (int c = tid; c < W; c += NT) st1(cr + c, xr[c] * rs * a.gain[c]);  // this thread's own stores
  }
}

template <typename T>
void launch_join(const JoinArgs& a, int rows, int W, float* x, int ldx, T* xc, int ldc, hipStream_t s) {
  const bool vec = !((W | ldx | ldc | a.ldy1 | a.ldg1 | a.ldg2 | a.ldy2 | a.ldye) % 4) &&
                   !(((uintptr_t)x | (uintptr_t)xc | (uintptr_t)a.y1 | (uintptr_t)a.g1 | (uintptr_t)a.g2 |
                      (uintptr_t)a.y2 | (uintptr_t)a.ye | (uintptr_t)a.gain) % 16);
  const int nv = vec ? (W + 1023) / 1024 : 0;
#define LSA_J(NV, NT) join_kernel<T, NV, NT><<<rows, NT, 0, s>>>(a, W, x, ldx, xc, ldc)
  if (nv >= 1 && nv <= 8 && rows <= 256) {  // few rows: their latency counts
    if (nv == 1) LSA_J(1, 256);
    else if (nv <= 4) LSA_J(1, 1024);
    else LSA_J(2, 1024);
  } else if (nv >= 1 && nv <= 2) LSA_J(2, 256);
  else if (nv >= 3 && nv <= 4) LSA_J(4, 256);
  else if (nv >= 5 && nv <= 8) LSA_J(8, 256);
  else LSA_J(0, 256);
#undef LSA_J
}

struct RenormArgs {  // Mirrored by llm_sharding_amd/ops/stream.py::RenormArgs
  const float* y;        // [rows][ldy] or null
  const void* ye;        // [rows * top][ldye] expert results of the sorted pairs, or null
  const float* weight;   // [rows * top]
  const int* place;      // [rows * top] where a row's pair lies in ye
  const float* post;     // norm of the result; null: as it is
  const float* gain;     // norm of the stream; null: the stream itself goes to the copy
  int ldy, ldye, top;
  int add;               // 0: the result takes the stream's place
  float eps;
};

// the result at [row][c .. c + V)
template <typename T, int V>
LSA_DEVICE void renorm_at(const RenormArgs& a, int row, int c, float* y) {
  if (a.y) {
    get<V>(a.y + (size_t)row * a.ldy + c, y);
  } else {
#pragma unroll
    for (int k = 0; k < V; ++k) y[k] = 0.f;
  }
  if (a.ye) add_pairs<V>((const T*)a.ye, a.ldye, a.weight, a.place, a.top, row, c, y);
}

// NT threads per row. NV > 0: rows of up to 4 NT NV values in registers, four at a time; 0: any width
template <typename T, int NV, int NT>
__global__ __launch_bounds__(NT) void renorm_kernel(RenormArgs a, int W, float* __restrict__ x, int ldx,
                                                     T* __restrict__ xc, int ldc) {
  __shared__ float s_part[NT / 64];
  const int row = blockIdx.x, tid = threadIdx.x;
  float* xr = x + (size_t)row * ldx;
  T* cr = xc + (size_t)row * ldc;
  if constexpr (NV > 0) {
    f32x4_t v[NV], xv[NV];
    float s = 0.f;
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int c = (tid + j * NT) * 4;
      v[j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
      xv[j] = v[j];
      if (c >= W) continue;
      if (a.add) xv[j] = *reinterpret_cast<const f32x4_t*>(xr + c);
      float f[4];
      renorm_at<T, 4>(a, row, c, f);
      v[j] = f32x4_t{f[0], f[1], f[2], f[3]};
#pragma unroll
      for (int k = 0; k < 4; ++k) s += f[k] * f[k];
    }
    float rs = 1.f;
    if (a.post) rs = 1.f / sqrtf(row_sum<NT>(s, s_part) / (float)W + a.eps);
    s = 0.f;
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int c = (tid + j * NT) * 4;
      if (c >= W) continue;
      if (a.post) v[j] = v[j] * rs * *reinterpret_cast<const f32x4_t*>(a.post + c);
      v[j] += xv[j];
      *reinterpret_cast<f32x4_t*>(xr + c) = v[j];
#pragma unroll
      for (int k = 0; k < 4; ++k) s += v[j][k] * v[j][k];
    }
    if (!xc) return;
    rs = 1.f;
    if (a.gain) rs = 1.f / sqrtf(row_sum<NT>(s, s_part) / (float)W + a.eps);
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int c = (tid + j * NT) * 4;
      if (c < W) st4(cr + c, a.gain ? v[j] * rs * *reinterpret_cast<const f32x4_t*>(a.gain + c) : v[j]);
    }
  } else {
    float s = 0.f, rs = 1.f;
    if (a.post) {
      for (int c = tid; c < W; c += NT) {
        float f;
        renorm_at<T, 1>(a, row, c, &f);
        s += f * f;
      }
      rs = 1.f / sqrtf(row_sum<NT>(s, s_part) / (float)W + a.eps);
    }
    s = 0.f;
    for (int c = tid; c < W; c += NT) {
      float f;
      renorm_at<T, 1>(a, row, c, &f);
      if (a.post) f *= rs * a.post[c];
      f += a.add ? xr[c] : 0.f;
      xr[c] = f;
      s += f * f;
    }
    if (!xc) return;
    rs = 1.f;
    if (a.gain) rs = 1.f / sqrtf(row_sum<NT>(s, s_part) / (float)W + a.eps);
    for (int c = tid; c < W; c += NT) st1(cr + c, a.gain ? xr[c] * rs * a.gain[c] : xr[c]);  // this thread's own stores
  }
}

template <typename T>
void launch_renorm(const RenormArgs& a, int rows, int W, float* x, int ldx, T* xc, int ldc, hipStream_t s) {
  const bool vec = !((W | ldx | ldc | a.ldy | a.ldye) % 4) &&
                   !(((uintptr_t)x | (uintptr_t)xc | (uintptr_t)a.y | (uintptr_t)a.ye | (uintptr_t)a.post |
                      (uintptr_t)a.gain) % 16);
  const int nv = vec ? (W + 1023) / 1024 : 0;
#define LSA_J(NV, NT) renorm_kernel<T, NV, NT><<<rows, NT, 0, s>>>(a, W, x, ldx, xc, ldc)
  if (nv >= 1 && nv <= 8 && rows <= 256) {  // few rows: their latency counts
    if (nv == 1) LSA_J(1, 256);
    else if (nv <= 4) LSA_J(1, 1024);
    else LSA_J(2, 1024);
  } else if (nv >= 1 && nv <= 2) LSA_J(2, 256);
  else if (nv >= 3 && nv <= 4) LSA_J(4, 256);
  else if (nv >= 5 && nv <= 8) LSA_J(8, 256);
  else LSA_J(0, 256);
#undef LSA_J
}

__global__ __launch_bounds__(256) void softcap_kernel(float* __restrict__ lg, int ldl, int n, float cap) {
  float* r = lg + (size_t)blockIdx.y * ldl;
  for (int c = blockIdx.x * 1024 + threadIdx.x; c < min(n, (int)(blockIdx.x + 1) * 1024); c += 256) r[c] = cap * tanhf(r[c] / cap);
}

// grid (rows, blocks): every workgroup one stretch of the vocabulary
__global__ __launch_bounds__(256) void logits_argmax_kernel(const float* __restrict__ lg, int ldl, int V, int offset,
                                                            unsigned long long* __restrict__ keys) {
  __shared__ unsigned long long s_key;
  if (threadIdx.x == 0) s_key = 0ull;
  __syncthreads();
  unsigned long long best = 0ull;
  for (int c = blockIdx.y * 256 + threadIdx.x; c < V; c += gridDim.y * 256) {
    const unsigned long long k = argmax_key(lg[(size_t)blockIdx.x * ldl + c], (unsigned)(c + offset));
    best = k > best ? k : best;
  }
  atomicMax(&s_key, best);
  __syncthreads();
  if (threadIdx.x == 0) atomicMax(keys + blockIdx.x, s_key);
}

}  // namespace

extern "C" int lsa_stream_embed(int f32, const int* ids, int rows, const void* table, int ldt, float scale, int W, int copies,
                                float* x, int ldx, void* xc, int ldc, hipStream_t s) {
  if (rows < 1 || W < 1 || copies < 1 || ldt < W || ldx < W * copies || (xc && ldc < W)) return LSA_BAD_SHAPE;
  if (f32)
    stream_embed_kernel<float><<<rows, 256, 0, s>>>(ids, (const float*)table, ldt, scale, W, copies, x, ldx, (float*)xc, ldc);
  else if (!((W | ldt | ldx | ldc) % 8) && !(((uintptr_t)table | (uintptr_t)x | (uintptr_t)xc) % 16))
    stream_embed8_kernel<<<rows, 256, 0, s>>>(ids, (const bf16_raw*)table, ldt, scale, W, copies, x, ldx, (bf16_raw*)xc, ldc);
  else
    stream_embed_kernel<bf16_raw><<<rows, 256, 0, s>>>(ids, (const bf16_raw*)table, ldt, scale, W, copies, x, ldx, (bf16_raw*)xc,
                                                       ldc);
  LSA_CHECK_LAUNCH();
  return LSA_OK;
}

extern "C" int lsa_cast_rows(int f32, const float* x, int ldx, int rows, int W, void* xc, int ldc, float* x2, int ldx2,
                             hipStream_t s) {
  if (rows < 1 || W < 1 || ldx < W || ldc < W || (x2 && ldx2 < W)) return LSA_BAD_SHAPE;
  const bool vec = !((W | ldx | ldc | ldx2) % 4) && !(((uintptr_t)x | (uintptr_t)xc | (uintptr_t)x2) % 16);
#define LSA_R(T, V) cast_rows_kernel<T, V><<<rows, 256, 0, s>>>(x, ldx, W, (T*)xc, ldc, x2, ldx2)
  if (f32 && vec) LSA_R(float, true);
  else if (f32) LSA_R(float, false);
  else if (vec) LSA_R(bf16_raw, true);
  else LSA_R(bf16_raw, false);
#undef LSA_R
  LSA_CHECK_LAUNCH();
  return LSA_OK;
}

extern "C" int lsa_stream_add_norm(int f32, const float* y, int ldy, const float* gain, float eps, int rows, int W,
                                   float* x, int ldx, void* xc, int ldc, hipStream_t s) {
  if (rows < 1 || W < 1 || ldy < W || ldx < W || ldc < W || !x) return LSA_BAD_SHAPE;
  if (f32) launch_norm<float, true>(y, ldy, gain, eps, rows, W, x, ldx, (float*)xc, ldc, s);
  else launch_norm<bf16_raw, true>(y, ldy, gain, eps, rows, W, x, ldx, (bf16_raw*)xc, ldc, s);
  LSA_CHECK_LAUNCH();
  return LSA_OK;
}

extern "C" int lsa_stream_norm(int f32, const float* y, int ldy, const float* gain, float eps, int rows, int W, void* xc,
                               int ldc, hipStream_t s) {
  if (rows < 1 || W < 1 || ldy < W || ldc < W) return LSA_BAD_SHAPE;
  if (f32) launch_norm<float, false>(y, ldy, gain, eps, rows, W, nullptr, 0, (float*)xc, ldc, s);
  else launch_norm<bf16_raw, false>(y, ldy, gain, eps, rows, W, nullptr, 0, (bf16_raw*)xc, ldc, s);
  LSA_CHECK_LAUNCH();
  return LSA_OK;
}

extern "C" int lsa_stream_join(int f32, const JoinArgs* a, int rows, int W, float* x, int ldx, void* xc, int ldc,
                               hipStream_t s) {
  if (!a || rows < 1 || W < 1 || ldx < W || !x || (a->gain && (!xc || ldc < W)) || (a->y2 && a->ye)) return LSA_BAD_SHAPE;
  if (a->y1 && (a->ldy1 < W || !a->g1 || a->ldg1 < W)) return LSA_BAD_SHAPE;
  if ((a->y2 || a->ye) && (!a->g2 || a->ldg2 < W)) return LSA_BAD_SHAPE;
  if (a->y2 && a->ldy2 < W) return LSA_BAD_SHAPE;
  if (a->ye && (a->ldye < W || a->top < 1 || !a->weight || !a->place)) return LSA_BAD_SHAPE;
  if (f32) launch_join<float>(*a, rows, W, x, ldx, (float*)xc, ldc, s);
  else launch_join<bf16_raw>(*a, rows, W, x, ldx, (bf16_raw*)xc, ldc, s);
  LSA_CHECK_LAUNCH();
  return LSA_OK;
}

extern "C" int lsa_stream_renorm(int f32, const RenormArgs* a, int rows, int W, float* x, int ldx, void* xc, int ldc,
                                 hipStream_t s) {
  if (!a || rows < 1 || W < 1 || ldx < W || !x || (xc && ldc < W) || (a->gain && !xc) || (!a->y && !a->ye)) return LSA_BAD_SHAPE;
  if (a->y && a->ldy < W) return LSA_BAD_SHAPE;
  if (a->ye && (a->ldye < W || a->top < 1 || !a->weight || !a->place)) return LSA_BAD_SHAPE;
  if (f32) launch_renorm<float>(*a, rows, W, x, ldx, (float*)xc, ldc, s);
  else launch_renorm<bf16_raw>(*a, rows, W, x, ldx, (bf16_raw*)xc, ldc, s);
  LSA_CHECK_LAUNCH();
  return LSA_OK;
}

extern "C" int lsa_softcap_rows(float* lg, int ldl, int rows, int n, float cap, hipStream_t s) {
  if (!lg || rows < 1 || rows > 65535 || n < 1 || ldl < n || !(cap > 0.f)) return LSA_BAD_SHAPE;
  softcap_kernel<<<dim3((n + 1023) / 1024, rows), 256, 0, s>>>(lg, ldl, n, cap);
  LSA_CHECK_LAUNCH();
  return LSA_OK;
}

extern "C" int lsa_logits_argmax(const float* lg, int ldl, int rows, int V, int offset, unsigned long long* keys,
                                 hipStream_t s) {
  if (rows < 1 || V < 1 || ldl < V || !keys) return LSA_BAD_SHAPE;
  logits_argmax_kernel<<<dim3(rows, (V + 4095) / 4096), 256, 0, s>>>(lg, ldl, V, offset, keys);
  LSA_CHECK_LAUNCH();
  return LSA_OK;
}
