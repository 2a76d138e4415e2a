// The gated delta rule step by step (delta.h): one workgroup per (run, head) keeps the head's state in
// registers and walks the run's rows; everything between the projections and the output projection in
// one launch. Decoded tokens are runs of one row; the fp32 engine runs whole portions this way.
#include "delta.h"

namespace {

// A row's vectors of one head in LDS: q, k (not yet of unit length), v, decays
template <typename T>
LSA_DEVICE void delta_row(const DeltaArgs& a, const DeltaRun& r, int t, int h, int channels, int DK, int DV, float* sq,
                          float* sk, float* sv, float* sg) {
  const int kb = h / (a.heads / a.kv_heads), kc = a.kv_heads * a.dim;
  for (int c = threadIdx.x; c < 2 * DK + DV; c += 256) {
    float x = 0.f;
    if (c < 2 * DK) {
      const int d = c < DK ? c : c - DK;
      if (d < a.dim)
        x = delta_conv<T>(a, r, t, (c < DK ? 0 : kc) + kb * a.dim + d, (c < DK ? a.oq : a.ok) + kb * a.dim + d, channels);
      (c < DK ? sq : sk)[d] = x;
    } else {
      const int d = c - 2 * DK;
      if (d < a.vdim) x = delta_conv<T>(a, r, t, 2 * kc + h * a.vdim + d, a.ov + h * a.vdim + d, channels);
      sv[d] = x;
    }
  }
  for (int d = threadIdx.x; d < DK; d += 256) sg[d] = d < a.dim ? expf(delta_log_decay(a, r.row0 + t, h, d)) : 0.f;
}

// sums of squares of q (wave 0) and k (wave 1) -> s[0], s[1]: what makes them unit vectors
LSA_DEVICE void delta_unit(const DeltaArgs& a, int DK, const float* sq, const float* sk, float* s) {
  const int w = threadIdx.x >> 6, lane = threadIdx.x & 63;
  if (w < 2) {
    const float* x = w ? sk : sq;
    float ss = 0.f;
    for (int d = lane; d < DK; d += 64) ss = fmaf(x[d], x[d], ss);
    ss = wave_sum(ss);
    if (lane == 0) s[w] = (w ? 1.f : a.q_scale) / sqrtf(ss + a.unit_eps);
  }
}

// the inputs of a one-row run join the ring: q and k by the first head that shares them
template <typename T>
LSA_DEVICE void delta_keep(const DeltaArgs& a, const DeltaRun& r, int h, int channels) {
  const int grp = a.heads / a.kv_heads, kb = h / grp, kc = a.kv_heads * a.dim;
  const T* in = (const T*)a.in + (size_t)r.row0 * a.ldi;
  float* ring = a.ring + ((size_t)r.slot * a.taps + r.pos0 % a.taps) * channels;
  for (int d = threadIdx.x; d < a.vdim; d += 256) ring[2 * kc + h * a.vdim + d] = ld1(in + a.ov + h * a.vdim + d);
  if (h % grp == 0)
    for (int d = threadIdx.x; d < a.dim; d += 256) {
      ring[kb * a.dim + d] = ld1(in + a.oq + kb * a.dim + d);
      ring[kc + kb * a.dim + d] = ld1(in + a.ok + kb * a.dim + d);
    }
}

template <typename T>
LSA_DEVICE void delta_store(const DeltaArgs& a, int row, int h, int d, float o, float rs) {
  float g = 1.f;
  if (a.gate) g = 1.f / (1.f + expf(-ld1((const T*)a.gate + (size_t)row * a.ldg + h * a.vdim + d)));
  st1((T*)a.out + (size_t)row * a.ldo + h * a.vdim + d, o * rs * a.norm[d] * g);
}

template <typename T, int DK, int DV>
__global__ __launch_bounds__(256) void delta_steps_kernel(DeltaArgs a, int keep) {
  // a thread holds RPT rows x 4 value channels of the state
  constexpr int NG = 1024 / DV, RPT = DK / NG;
  static_assert(RPT >= 1 && NG * RPT == DK, "geometry");
  __shared__ __attribute__((aligned(16))) float sq[DK], sk[DK], sg[DK], sv[DV], s_a[NG][DV], s_b[NG][DV];
  __shared__ float s_unit[2], s_ss[4];
  const DeltaRun r = delta_run(a, blockIdx.x);
  const int h = blockIdx.y, tid = threadIdx.x, v = (tid % (DV / 4)) * 4, grp = tid / (DV / 4), d0 = grp * RPT;
  const int channels = 2 * a.kv_heads * a.dim + a.heads * a.vdim;
  if (r.n == 0) {
    if (!a.runs)
      for (int d = tid; d < a.vdim; d += 256) st1((T*)a.out + (size_t)r.row0 * a.ldo + h * a.vdim + d, 0.f);
    return;
  }
  float* st = a.state + ((size_t)r.slot * a.heads + h) * DK * DV + (size_t)d0 * DV + v;
  f32x4_t S[RPT];
#pragma unroll
  for (int j = 0; j < RPT; ++j) S[j] = *reinterpret_cast<const f32x4_t*>(st + (size_t)j * DV);
  if (r.pos0 == 0) {
#pragma unroll
    for (int j = 0; j < RPT; ++j) S[j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  }
  for (int t = 0; t < r.n; ++t) {
    const int row = r.row0 + t;
    delta_row<T>(a, r, t, h, channels, DK, DV, sq, sk, sv, sg);
    __syncthreads();
    delta_unit(a, DK, sq, sk, s_unit);
    f32x4_t part = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int j = 0; j < RPT; ++j) {
      S[j] *= sg[d0 + j];
      part += S[j] * sk[d0 + j];
    }
    *reinterpret_cast<f32x4_t*>(&s_a[grp][v]) = part;
    __syncthreads();
    const float ku = s_unit[1], beta = 1.f / (1.f + expf(-a.in32[(size_t)row * a.ld32 + a.ob + h]));
    f32x4_t dot = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int g = 0; g < NG; ++g) dot += *reinterpret_cast<const f32x4_t*>(&s_a[g][v]);
    // beta (v - S^T k), times the scale of k
    const f32x4_t u = (*reinterpret_cast<const f32x4_t*>(&sv[v]) - dot * ku) * (beta * ku);
    f32x4_t o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int j = 0; j < RPT; ++j) {
      S[j] += u * sk[d0 + j];
      o += S[j] * sq[d0 + j];
    }
    *reinterpret_cast<f32x4_t*>(&s_b[grp][v]) = o;
    __syncthreads();
    float x = 0.f;
    if (tid < DV) {
#pragma unroll
      for (int g = 0; g < NG; ++g) x += s_b[g][tid];
      x *= s_unit[0];
    }
    const float ss = wave_sum(x * x);
    if ((tid & 63) == 0) s_ss[tid >> 6] = ss;
    __syncthreads();
    if (tid < a.vdim) delta_store<T>(a, row, h, tid, x, 1.f / sqrtf((s_ss[0] + s_ss[1] + s_ss[2] + s_ss[3]) / (float)a.vdim + a.eps));
  }
#pragma unroll
  for (int j = 0; j < RPT; ++j) *reinterpret_cast<f32x4_t*>(st + (size_t)j * DV) = S[j];
  if (keep) delta_keep<T>(a, r, h, channels);
}

// any size: the state stays in memory; thread <-> value channels
template <typename T>
__global__ __launch_bounds__(256) void delta_plain_kernel(DeltaArgs a, int keep) {
  extern __shared__ float smem[];
  const int DK = a.dk, DV = a.dv, tid = threadIdx.x, h = blockIdx.y;
  float *sq = smem, *sk = sq + DK, *sg = sk + DK, *sv = sg + DK, *so = sv + DV;
  __shared__ float s_unit[2], s_ss[4];
  const DeltaRun r = delta_run(a, blockIdx.x);
  const int channels = 2 * a.kv_heads * a.dim + a.heads * a.vdim;
  if (r.n == 0) {
    if (!a.runs)
      for (int d = tid; d < a.vdim; d += 256) st1((T*)a.out + (size_t)r.row0 * a.ldo + h * a.vdim + d, 0.f);
    return;
  }
  float* st = a.state + ((size_t)r.slot * a.heads + h) * DK * DV;
  for (int t = 0; t < r.n; ++t) {
    const int row = r.row0 + t;
    const bool fresh = t == 0 && r.pos0 == 0;
    __syncthreads();
    delta_row<T>(a, r, t, h, channels, DK, DV, sq, sk, sv, sg);
    __syncthreads();
    delta_unit(a, DK, sq, sk, s_unit);
    __syncthreads();
    const float ku = s_unit[1], beta = 1.f / (1.f + expf(-a.in32[(size_t)row * a.ld32 + a.ob + h]));
    float ss = 0.f;
    for (int v = tid; v < DV; v += 256) {
      float dot = 0.f;
      for (int d = 0; d < DK; ++d) {
        const float x = fresh ? 0.f : st[(size_t)d * DV + v] * sg[d];
        st[(size_t)d * DV + v] = x;
        dot = fmaf(x, sk[d], dot);
      }
      const float u = beta * (sv[v] - dot * ku) * ku;
      float o = 0.f;
      for (int d = 0; d < DK; ++d) {
        const float x = fmaf(sk[d], u, st[(size_t)d * DV + v]);
        st[(size_t)d * DV + v] = x;
        o = fmaf(x, sq[d], o);
      }
      o *= s_unit[0];
      so[v] = o;
      ss = fmaf(o, o, ss);
    }
    ss = wave_sum(ss);
    if ((tid & 63) == 0) s_ss[tid >> 6] = ss;
    __syncthreads();
    const float rs = 1.f / sqrtf((s_ss[0] + s_ss[1] + s_ss[2] + s_ss[3]) / (float)a.vdim + a.eps);
    for (int d = tid; d < a.vdim; d += 256) delta_store<T>(a, row, h, d, so[d], rs);
  }
  if (keep) delta_keep<T>(a, r, h, channels);
}

// the last inputs of every run join its slot's ring (after everything that reads the ring)
template <typename T>
__global__ __launch_bounds__(256) void delta_ring_kernel(DeltaArgs a) {
  const DeltaRun r = delta_run(a, blockIdx.x);
  const int kc = a.kv_heads * a.dim, channels = 2 * kc + a.heads * a.vdim, n = min(r.n, a.taps);
  for (int c = blockIdx.y * 256 + threadIdx.x; c < channels; c += gridDim.y * 256) {
    const int col = c < kc ? a.oq + c : (c < 2 * kc ? a.ok + c - kc : a.ov + c - 2 * kc);
    for (int t = r.n - n; t < r.n; ++t)
      a.ring[((size_t)r.slot * a.taps + (r.pos0 + t) % a.taps) * channels + c] =
          ld1((const T*)a.in + (size_t)(r.row0 + t) * a.ldi + col);
  }
}

}  // namespace

// n runs (a->runs), or n single rows (a->slot / a->pos). keep: every run is one row and joins the ring
// here; else lsa_delta_ring follows
extern "C" int lsa_delta_steps(int f32, const DeltaArgs* a, int n, int keep, hipStream_t s) {
  if (bad_delta(a) || n < 1) return LSA_BAD_SHAPE;
  const dim3 grid(n, a->heads);
#define LSA_D(K, V)                                                                 \
  if (a->dk == K && a->dv == V) {                                                   \
    if (f32) delta_steps_kernel<float, K, V><<<grid, 256, 0, s>>>(*a, keep);        \
    else delta_steps_kernel<bf16_raw, K, V><<<grid, 256, 0, s>>>(*a, keep);         \
    LSA_CHECK_LAUNCH();                                                             \
    return LSA_OK;                                                                  \
  }
  LSA_D(32, 32) LSA_D(32, 64) LSA_D(32, 128) LSA_D(64, 32) LSA_D(64, 64) LSA_D(64, 128) LSA_D(128, 32) LSA_D(128, 64)
  LSA_D(128, 128)
#undef LSA_D
  const size_t lds = (size_t)(3 * a->dk + 2 * a->dv) * 4;
  if (lds > 60000) return LSA_UNSUPPORTED;
  if (f32) delta_plain_kernel<float><<<grid, 256, lds, s>>>(*a, keep);
  else delta_plain_kernel<bf16_raw><<<grid, 256, lds, s>>>(*a, keep);
  LSA_CHECK_LAUNCH();
  return LSA_OK;
}

extern "C" int lsa_delta_ring(int f32, const DeltaArgs* a, int n, hipStream_t s) {
  if (bad_delta(a) || n < 1) return LSA_BAD_SHAPE;
  const int channels = 2 * a->kv_heads * a->dim + a->heads * a->vdim;
  const dim3 grid(n, (channels + 255) / 256);
  if (f32) delta_ring_kernel<float><<<grid, 256, 0, s>>>(*a);
  else delta_ring_kernel<bf16_raw><<<grid, 256, 0, s>>>(*a);
  LSA_CHECK_LAUNCH();
  return LSA_OK;
}
