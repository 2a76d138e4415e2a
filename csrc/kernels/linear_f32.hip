// Projections of the fp32 engine: C[M][N] = A[M][K] . W[N][K]^T with true fp32 products and sums
// (VALU FMA; no reduced-precision matrix mode). 64 x 64 tiles, 16-deep K steps through LDS, 4 x 4
// outputs per thread. Epilogues: store, or the gated unit over interleaved 16-row gate / up
// blocks (ops/packing.py fuse_gate_up), as EPI_STORE / EPI_SWIGLU / EPI_GEGLU of the bf16 GEMMs.
#include "epilogue.h"

namespace {

constexpr int TM = 64, TN = 64, TK = 16;

// epi_store1 with fp32 in the place of bf16 (ep.out, ep.gate)
LSA_DEVICE void store_f32(const EpiArgs& ep, int m, int n, float v) {
  v += epi_bias(ep, n);
  if (ep.act && epi_acts(ep, n)) v = epi_activate(ep.act, v);
  if (!ep.out32 || n < ep.col32) {
    ((float*)ep.out)[(size_t)m * ep.ldo + n] = v;
    return;
  }
  float* o = ep.out32 + (size_t)m * ep.ldo32 + (n - ep.col32);
  if (!ep.gate) *o = v;
  else if (n < ep.cols) *o += sigmoid(((const float*)ep.gate)[(size_t)m * ep.ldg + n]) * v;
}

template <int EPI>
__global__ __launch_bounds__(256) void linear_f32_kernel(const float* __restrict__ A, int lda,
                                                         const float* __restrict__ W, int M, int N, int K, EpiArgs ep) {
  __shared__ float sa[TK][TM + 4], sw[TK][TN + 4];
  const int tid = threadIdx.x, n0 = blockIdx.x * TN, m0 = blockIdx.y * TM;
  // thread -> rows m0 + ty + 16 i, columns n0 + tx + 16 j: with GLU, columns tx + 16 (2p) and
  // tx + 16 (2p + 1) are the gate and the up value of one output
  const int tx = tid & 15, ty = tid >> 4;
  const int lr = tid >> 2, lk = (tid & 3) * 4;
  float acc[4][4];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = 0.f;
  const float* ar = A + (size_t)min(m0 + lr, M - 1) * lda;  // rows past M are computed and not stored
  const float* wr = W + (size_t)min(n0 + lr, N - 1) * K;
  for (int k0 = 0; k0 < K; k0 += TK) {  // K % 16 == 0
    const f32x4_t a = *reinterpret_cast<const f32x4_t*>(ar + k0 + lk);
    const f32x4_t w = *reinterpret_cast<const f32x4_t*>(wr + k0 + lk);
    __syncthreads();
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      sa[lk + q][lr] = a[q];
      sw[lk + q][lr] = w[q];
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < TK; ++k) {
      float av[4], wv[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) av[i] = sa[k][ty + 16 * i];
#pragma unroll
      for (int j = 0; j < 4; ++j) wv[j] = sw[k][tx + 16 * j];
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = fmaf(av[i], wv[j], acc[i][j]);
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int m = m0 + ty + 16 * i;
    if (m >= M) continue;
    if constexpr (epi_gated(EPI)) {
#pragma unroll
      for (int p = 0; p < 2; ++p) {
        const int c = n0 + 32 * p;
        if (c >= N) continue;
        const int n = c + tx;
        ep.out32[(size_t)m * ep.ldo + c / 2 + tx] =
            epi_glu<EPI>(ep, acc[i][2 * p] + epi_bias(ep, n), acc[i][2 * p + 1] + epi_bias(ep, n + 16));
      }
    } else {
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int n = n0 + tx + 16 * j;
        if (n < N) store_f32(ep, m, n, acc[i][j]);
      }
    }
  }
}

}  // namespace

extern "C" int lsa_linear_f32(const float* a, int lda, const float* w, int M, int N, int K, int epi, const EpiArgs* ep,
                              hipStream_t stream) {
  if (M < 1 || N < 1 || K < 16 || K % 16 || lda < K || lda % 4 || !ep || !(ep->out32 || ep->out)) return LSA_BAD_SHAPE;
  if (((uintptr_t)a | (uintptr_t)w) % 16) return LSA_BAD_SHAPE;
  dim3 grid((N + TN - 1) / TN, (M + TM - 1) / TM);
  if (epi_gated(epi)) {
    if (N % 32 || ep->ldo < N / 2 || !ep->out32) return LSA_BAD_SHAPE;
    if (epi == EPI_GEGLU) linear_f32_kernel<EPI_GEGLU><<<grid, 256, 0, stream>>>(a, lda, w, M, N, K, *ep);
    else linear_f32_kernel<EPI_SWIGLU><<<grid, 256, 0, stream>>>(a, lda, w, M, N, K, *ep);
  } else if (epi == EPI_STORE) {
    if (bad_store(*ep, N)) return LSA_BAD_SHAPE;
    linear_f32_kernel<EPI_STORE><<<grid, 256, 0, stream>>>(a, lda, w, M, N, K, *ep);
  } else {
    return LSA_UNSUPPORTED;
  }
  LSA_CHECK_LAUNCH();
  return LSA_OK;
}
