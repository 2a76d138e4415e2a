// Several residual streams side by side (hyper-connections): a row is [streams][width] in fp32.
//
//   lsa_stream_mix  x_t <- sum_s mix[s][t] x_s + out[t] v of a sublayer's result v (every stream from all old
//                   ones), then (optionally) rms(sum_s in[s] x_s) * gain -> the next sublayer's input. v is an fp32
//                   result, times the sigmoid of a number per row, and / or the weighted sum of a row's expert results
//
// One pass over the row: a thread has the same columns of all streams, so the next input's norm costs no second read.
#include "stream_row.h"

namespace {

constexpr int MAXS = 16;

struct MixArgs {  // Mirrored by llm_sharding_amd/ops/stream.py::MixArgs
  const float* coef;     // [streams] out, [streams][streams] mix (from, to); null: the streams stay
  const float* y;        // [rows][ldy] or null
  const float* ygate;    // [rows][ldyg] logit of y's gate, or null
  const void* ye;        // [rows * top][ldye] expert results of the sorted pairs, or null
  const float* weight;   // [rows * top]
  const int* place;      // [rows * top] where a row's pair lies in ye
  const float* read;     // [streams] in; null: nothing is read
  const float* gain;     // [width]
  int streams, ldy, ldyg, ldye, top;
  float eps;
};

// the result at [row][c .. c + V)
template <typename T, int V>
LSA_DEVICE void result_at(const MixArgs& a, int row, int c, float gate, float* y) {
#pragma unroll
  for (int k = 0; k < V; ++k) y[k] = 0.f;
  if (a.y) {
    get<V>(a.y + (size_t)row * a.ldy + c, y);
#pragma unroll
    for (int k = 0; k < V; ++k) y[k] *= gate;
  }
  if (a.ye) add_pairs<V>((const T*)a.ye, a.ldye, a.weight, a.place, a.top, row, c, y);
}

// V columns of all streams: mixed and stored; u = their weighted sum. S: streams, 0: any number up to MAXS
template <typename T, int S, int V>
LSA_DEVICE void mix_at(const MixArgs& a, int row, int c, int W, float* xr, float gate, float* u) {
  constexpr int M = S ? S : MAXS;
  const int n = S ? S : a.streams;
  float x[M][V];
#pragma unroll
  for (int s = 0; s < M; ++s)
    if (s < n) get<V>(xr + (size_t)s * W + c, x[s]);
#pragma unroll
  for (int k = 0; k < V; ++k) u[k] = 0.f;
  if (a.coef) {
    float y[V];
    result_at<T, V>(a, row, c, gate, y);
#pragma unroll
    for (int t = 0; t < M; ++t) {
      if (t >= n) continue;
      float z[V];
#pragma unroll
      for (int k = 0; k < V; ++k) z[k] = a.coef[t] * y[k];
#pragma unroll
      for (int s = 0; s < M; ++s) {
        if (s >= n) continue;
        const float m = a.coef[n + s * n + t];
#pragma unroll
        for (int k = 0; k < V; ++k) z[k] = fmaf(m, x[s][k], z[k]);
      }
      float* d = xr + (size_t)t * W + c;
      if constexpr (V == 4) *reinterpret_cast<f32x4_t*>(d) = f32x4_t{z[0], z[1], z[2], z[3]};
      else *d = z[0];
      if (a.read) {
        const float r = a.read[t];
#pragma unroll
        for (int k = 0; k < V; ++k) u[k] = fmaf(r, z[k], u[k]);
      }
    }
  } else {
#pragma unroll
    for (int s = 0; s < M; ++s) {
      if (s >= n) continue;
      const float r = a.read[s];
#pragma unroll
      for (int k = 0; k < V; ++k) u[k] = fmaf(r, x[s][k], u[k]);
    }
  }
}

// NT threads per row. NV > 0: the sums of rows of up to 4 NT NV columns stay in registers; 0: any width
template <typename T, int S, int NV, int NT>
__global__ __launch_bounds__(NT) void mix_kernel(MixArgs a, int W, float* __restrict__ x, int ldx, T* __restrict__ xc, int ldc) {
  __shared__ float s_part[NT / 64];
  const int row = blockIdx.x, tid = threadIdx.x;
  float* xr = x + (size_t)row * ldx;
  const float gate = a.ygate ? sigmoid(a.ygate[(size_t)row * a.ldyg]) : 1.f;
  float s = 0.f;
  if constexpr (NV > 0) {
    f32x4_t u[NV];
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int c = (tid + j * NT) * 4;
      u[j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
      if (c >= W) continue;
      float f[4];
      mix_at<T, S, 4>(a, row, c, W, xr, gate, f);
      u[j] = f32x4_t{f[0], f[1], f[2], f[3]};
#pragma unroll
      for (int k = 0; k < 4; ++k) s += f[k] * f[k];
    }
    if (!a.read) return;
    const float rs = 1.f / sqrtf(row_sum<NT>(s, s_part) / (float)W + a.eps);
    T* cr = xc + (size_t)row * ldc;
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int c = (tid + j * NT) * 4;
      if (c < W) st4(cr + c, u[j] * rs * *reinterpret_cast<const f32x4_t*>(a.gain + c));
    }
  } else {
    for (int c = tid; c < W; c += NT) {
      float f;
      mix_at<T, S, 1>(a, row, c, W, xr, gate, &f);
      s += f * f;
    }
    if (!a.read) return;
    const float rs = 1.f / sqrtf(row_sum<NT>(s, s_part) / (float)W + a.eps);
    T* cr = xc + (size_t)row * ldc;
    const int n = S ? S : a.streams;
    for (int c = tid; c < W; c += NT) {  // this thread's own stores
      float f = 0.f;
      for (int t = 0; t < n; ++t) f = fmaf(a.read[t], xr[(size_t)t * W + c], f);
      st1(cr + c, f * rs * a.gain[c]);
    }
  }
}

template <typename T, int S>
void launch_mix(const MixArgs& a, int rows, int W, float* x, int ldx, T* xc, int ldc, hipStream_t s) {
  const bool vec = !((W | ldx | ldc | a.ldy | a.ldye) % 4) &&
                   !(((uintptr_t)x | (uintptr_t)xc | (uintptr_t)a.y | (uintptr_t)a.ye | (uintptr_t)a.gain) % 16);
  const int nv = vec ? (W + 1023) / 1024 : 0;
#define LSA_M(NV, NT) mix_kernel<T, S, NV, NT><<<rows, NT, 0, s>>>(a, W, x, ldx, xc, ldc)
  if (nv >= 1 && nv <= 8 && rows <= 256) {  // few rows: their latency counts
    if (nv == 1) LSA_M(1, 256);
    else if (nv <= 4) LSA_M(1, 1024);
    else LSA_M(2, 1024);
  } else if (nv >= 1 && nv <= 2) LSA_M(2, 256);
  else if (nv >= 3 && nv <= 4) LSA_M(4, 256);
  else if (nv >= 5 && nv <= 8) LSA_M(8, 256);
  else LSA_M(0, 256);
#undef LSA_M
}

template <typename T>
void launch_streams(const MixArgs& a, int rows, int W, float* x, int ldx, T* xc, int ldc, hipStream_t s) {
  switch (a.streams) {
    case 1: launch_mix<T, 1>(a, rows, W, x, ldx, xc, ldc, s); break;
    case 2: launch_mix<T, 2>(a, rows, W, x, ldx, xc, ldc, s); break;
    case 3: launch_mix<T, 3>(a, rows, W, x, ldx, xc, ldc, s); break;
    case 4: launch_mix<T, 4>(a, rows, W, x, ldx, xc, ldc, s); break;
    default: launch_mix<T, 0>(a, rows, W, x, ldx, xc, ldc, s);
  }
}

}  // namespace

extern "C" int lsa_stream_mix(int f32, const MixArgs* a, int rows, int W, float* x, int ldx, void* xc, int ldc, hipStream_t s) {
  if (!a || rows < 1 || W < 1 || !x || a->streams < 1 || a->streams > MAXS || ldx < W * a->streams) return LSA_BAD_SHAPE;
  if (!a->coef && !a->read) return LSA_BAD_SHAPE;
  if ((a->coef != nullptr) != (a->y || a->ye)) return LSA_BAD_SHAPE;
  if ((a->y && a->ldy < W) || (a->ygate && !a->y)) return LSA_BAD_SHAPE;
  if (a->ye && (a->ldye < W || a->top < 1 || !a->weight || !a->place)) return LSA_BAD_SHAPE;
  if (a->read && (!a->gain || !xc || ldc < W)) return LSA_BAD_SHAPE;
  if (f32) launch_streams<float>(*a, rows, W, x, ldx, (float*)xc, ldc, s);
  else launch_streams<bf16_raw>(*a, rows, W, x, ldx, (bf16_raw*)xc, ldc, s);
  LSA_CHECK_LAUNCH();
  return LSA_OK;
}
