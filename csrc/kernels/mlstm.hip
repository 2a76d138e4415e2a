// Matrix memory step by step (mlstm.h): one workgroup per (run, head) keeps the head's state in registers and walks
// the run's rows; everything between the projections and the output projection in one launch. Decoded tokens are runs
// of one row; the fp32 engine runs whole portions this way.
#include "mlstm.h"

namespace {

template <typename T>
LSA_DEVICE void ml_row(const MlArgs& a, int row, int h, int DK, int DV, float* sq, float* sk, float* sv) {
  const T* in = (const T*)a.in + (size_t)row * a.ldi;
  for (int c = threadIdx.x; c < 2 * DK + DV; c += 256) {
    if (c < DK) sq[c] = ld1(in + a.oq + h * DK + c) * a.q_scale;
    else if (c < 2 * DK) sk[c - DK] = ld1(in + a.ok + h * DK + c - DK);
    else sv[c - 2 * DK] = ld1(in + a.ov + h * DV + c - 2 * DK);
  }
}

template <typename T>
LSA_DEVICE void ml_store(const MlArgs& a, int row, int h, int d, float o, float rs) {
  const float g = ld1((const T*)a.in + (size_t)row * a.ldi + a.og + h * a.dv + d);
  st1((T*)a.out + (size_t)row * a.ldo + h * a.dv + d, o * rs * a.norm[h * a.dv + d] * sigmoid(g));
}

template <typename T>
LSA_DEVICE bool ml_idle(const MlArgs& a, const MlRun& r, int h) {
  if (r.n) return false;
  if (!a.runs)
    for (int d = threadIdx.x; d < a.dv; d += 256) st1((T*)a.out + (size_t)r.row0 * a.ldo + h * a.dv + d, 0.f);
  return true;
}

template <typename T, int DK, int DV>
__global__ __launch_bounds__(256) void ml_steps_kernel(MlArgs a) {
  // a thread holds RPT rows x 4 value channels of S and the same rows of n
  constexpr int NG = 1024 / DV, RPT = DK / NG;
  static_assert(RPT >= 1 && NG * RPT == DK, "geometry");
  __shared__ __attribute__((aligned(16))) float sq[DK], sk[DK], sv[DV], s_b[NG][DV], s_n[NG];
  __shared__ float s_ss[4];
  const MlRun r = ml_run(a, blockIdx.x);
  const int h = blockIdx.y, tid = threadIdx.x, v = (tid % (DV / 4)) * 4, grp = tid / (DV / 4), d0 = grp * RPT;
  if (ml_idle<T>(a, r, h)) return;
  const size_t head = (size_t)r.slot * a.heads + h;
  float* st = a.S + head * DK * DV + (size_t)d0 * DV + v;
  float* sn = a.n + head * a.copies * DK;
  f32x4_t S[RPT];
  float n[RPT], m = a.m[head * a.copies];
#pragma unroll
  for (int j = 0; j < RPT; ++j) {
    S[j] = *reinterpret_cast<const f32x4_t*>(st + (size_t)j * DV);
    n[j] = sn[d0 + j];
  }
  if (r.pos0 == 0) {
#pragma unroll
    for (int j = 0; j < RPT; ++j) {
      S[j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
      n[j] = 0.f;
    }
    m = 0.f;
  }
  for (int t = 0; t < r.n; ++t) {
    const int row = r.row0 + t;
    ml_row<T>(a, row, h, DK, DV, sq, sk, sv);
    const float i = ml_input_gate(a, row, h), fm = ml_forget_gate(a, row, h) + m;
    m = fmaxf(fm, i);
    const float keep = expf(fm - m), add = expf(i - m);
    __syncthreads();
    const f32x4_t u = *reinterpret_cast<const f32x4_t*>(&sv[v]) * add;
    f32x4_t o = {0.f, 0.f, 0.f, 0.f};
    float nq = 0.f;
#pragma unroll
    for (int j = 0; j < RPT; ++j) {
      const float k = sk[d0 + j], q = sq[d0 + j];
      S[j] = S[j] * keep + u * k;
      o += S[j] * q;
      n[j] = n[j] * keep + add * k;
      nq += n[j] * q;
    }
    *reinterpret_cast<f32x4_t*>(&s_b[grp][v]) = o;
    if (v == 0) s_n[grp] = nq;
    __syncthreads();
    float x = 0.f;
    if (tid < DV) {
      float z = 0.f;
#pragma unroll
      for (int g = 0; g < NG; ++g) {
        x += s_b[g][tid];
        z += s_n[g];
      }
      x /= ml_denominator(z, m);
    }
    const float ss = wave_sum(x * x);
    if ((tid & 63) == 0) s_ss[tid >> 6] = ss;
    __syncthreads();
    if (tid < DV) ml_store<T>(a, row, h, tid, x, 1.f / sqrtf((s_ss[0] + s_ss[1] + s_ss[2] + s_ss[3]) / (float)a.vdim + a.eps));
  }
#pragma unroll
  for (int j = 0; j < RPT; ++j) *reinterpret_cast<f32x4_t*>(st + (size_t)j * DV) = S[j];
  for (int c = 0; c < a.copies; ++c) {
    if (v == 0) {
#pragma unroll
      for (int j = 0; j < RPT; ++j) sn[(size_t)c * DK + d0 + j] = n[j];
    }
    if (tid == 0) a.m[head * a.copies + c] = m;
  }
}

// any size (one copy): the state stays in memory; thread <-> value channels, and key channels of n
template <typename T>
__global__ __launch_bounds__(256) void ml_plain_kernel(MlArgs a) {
  extern __shared__ float smem[];
  const int DK = a.dk, DV = a.dv, tid = threadIdx.x, h = blockIdx.y;
  float *sq = smem, *sk = sq + DK, *sv = sk + DK, *so = sv + DV;
  __shared__ float s_ss[4], s_n[4];
  const MlRun r = ml_run(a, blockIdx.x);
  if (ml_idle<T>(a, r, h)) return;
  const size_t head = (size_t)r.slot * a.heads + h;
  float *st = a.S + head * DK * DV, *sn = a.n + head * DK;
  float m = r.pos0 == 0 ? 0.f : a.m[head];
  for (int t = 0; t < r.n; ++t) {
    const bool fresh = t == 0 && r.pos0 == 0;
    const int row = r.row0 + t;
    __syncthreads();
    ml_row<T>(a, row, h, DK, DV, sq, sk, sv);
    const float i = ml_input_gate(a, row, h), fm = ml_forget_gate(a, row, h) + m;
    m = fmaxf(fm, i);
    const float keep = expf(fm - m), add = expf(i - m);
    __syncthreads();
    float nq = 0.f;
    for (int d = tid; d < DK; d += 256) {
      const float z = (fresh ? 0.f : sn[d] * keep) + add * sk[d];
      sn[d] = z;
      nq = fmaf(z, sq[d], nq);
    }
    nq = wave_sum(nq);
    if ((tid & 63) == 0) s_n[tid >> 6] = nq;
    __syncthreads();
    const float den = ml_denominator(s_n[0] + s_n[1] + s_n[2] + s_n[3], m);
    float ss = 0.f;
    for (int v = tid; v < DV; v += 256) {
      float o = 0.f;
      const float u = sv[v] * add;
      for (int d = 0; d < DK; ++d) {
        const float x = fmaf(sk[d], u, fresh ? 0.f : st[(size_t)d * DV + v] * keep);
        st[(size_t)d * DV + v] = x;
        o = fmaf(x, sq[d], o);
      }
      o /= den;
      so[v] = o;
      ss = fmaf(o, o, ss);
    }
    ss = wave_sum(ss);
    if ((tid & 63) == 0) s_ss[tid >> 6] = ss;
    __syncthreads();
    const float rs = 1.f / sqrtf((s_ss[0] + s_ss[1] + s_ss[2] + s_ss[3]) / (float)a.vdim + a.eps);
    for (int d = tid; d < DV; d += 256) ml_store<T>(a, row, h, d, so[d], rs);
  }
  if (tid == 0) a.m[head] = m;  // read before the first barrier
}

}  // namespace

// n runs (a->runs), or n single rows (a->slot / a->pos)
extern "C" int lsa_ml_steps(int f32, const MlArgs* a, int n, hipStream_t s) {
  if (bad_ml(a) || n < 1) return LSA_BAD_SHAPE;
  const dim3 grid(n, a->heads);
#define LSA_D(K, V)                                                   \
  if (a->dk == K && a->dv == V) {                                     \
    if (f32) ml_steps_kernel<float, K, V><<<grid, 256, 0, s>>>(*a);   \
    else ml_steps_kernel<bf16_raw, K, V><<<grid, 256, 0, s>>>(*a);    \
    LSA_CHECK_LAUNCH();                                               \
    return LSA_OK;                                                    \
  }
  LSA_D(32, 32) LSA_D(32, 64) LSA_D(32, 128) LSA_D(64, 32) LSA_D(64, 64) LSA_D(64, 128) LSA_D(128, 32) LSA_D(128, 64)
  LSA_D(128, 128)
#undef LSA_D
  if (a->copies != 1) return LSA_BAD_SHAPE;
  const size_t lds = (size_t)(2 * a->dk + 2 * a->dv) * 4;
  if (lds > 60000) return LSA_UNSUPPORTED;
  if (f32) ml_plain_kernel<float><<<grid, 256, lds, s>>>(*a);
  else ml_plain_kernel<bf16_raw><<<grid, 256, lds, s>>>(*a);
  LSA_CHECK_LAUNCH();
  return LSA_OK;
}
