// Latent attention, the steps every path shares and the plain form of the others (latent.h):
//   lsa_latent_append  normed query latent, normed key latent and rotated key part of a row, the
//                      last two appended to the paged cache
//   lsa_latent_absorb  q~ = W_uk^T q per head, and the rotated query part behind it
//   lsa_latent_attend  split softmax attention over the cache in the absorbed form
//   lsa_latent_value   merge of the splits, W_uv per head, output gate
//   lsa_latent_gather  a sequence's cached entries -> consecutive rows (the expanded form's input)
// The plain kernels (one workgroup per row and head, VALU) compute in the type of the engine and
// take every size; bf16 engines use the MFMA kernels of latent_decode.hip wherever those have the size.
#include "latent.h"

namespace {

// sum over the 256 threads of a workgroup
LSA_DEVICE float block_sum(float v, float* part) {
  v = wave_sum(v);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) part[threadIdx.x >> 6] = v;
  __syncthreads();
  return part[0] + part[1] + part[2] + part[3];
}
LSA_DEVICE float block_max(float v, float* part) {
  v = wave_max(v);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) part[threadIdx.x >> 6] = v;
  __syncthreads();
  return fmaxf(fmaxf(part[0], part[1]), fmaxf(part[2], part[3]));
}

// (a, b) summed over the 256 threads of a workgroup
LSA_DEVICE void block_sum2(float& a, float& b, float (*part)[4]) {
  a = wave_sum(a);
  b = wave_sum(b);
  if ((threadIdx.x & 63) == 0) {
    part[0][threadIdx.x >> 6] = a;
    part[1][threadIdx.x >> 6] = b;
  }
  __syncthreads();
  a = part[0][0] + part[0][1] + part[0][2] + part[0][3];
  b = part[1][0] + part[1][1] + part[1][2] + part[1][3];
}

LSA_DEVICE void ld8(const float* p, float* f) {
#pragma unroll
  for (int k = 0; k < 8; ++k) f[k] = p[k];
}
LSA_DEVICE void ld8(const bf16_raw* p, float* f) { unpack8(ld16(p), f); }
LSA_DEVICE void st8(float* p, const float* f) {
#pragma unroll
  for (int k = 0; k < 8; ++k) p[k] = f[k];
}
LSA_DEVICE void st8(bf16_raw* p, const float* f) { st16(p, pack8(f)); }

// in: row of the fused input projection, query latent at column oq, [key latent | rotated part] at
// ok. VEC: 8 values at a time (ranks and offsets multiples of 8), the first of a thread's stretches
// kept in registers between the sums and the scaling.
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void append_kernel(LatentArgs a, const T* __restrict__ in, int ldi, int oq, int ok,
                                                     const float* __restrict__ gq, const float* __restrict__ gk,
                                                     T* __restrict__ cq, int ldc) {
  __shared__ float part[2][4];
  constexpr int S = VEC ? 8 : 1;
  const int row = blockIdx.x, tid = threadIdx.x;
  const T* q = in + (size_t)row * ldi + oq;
  const T* k = in + (size_t)row * ldi + ok;
  const int nq = a.q_rank / S, n = nq + a.kv_rank / S;  // stretches of both latents
  float sq = 0.f, sk = 0.f, first[S];
  auto load = [&](int c, float* f) {
    const T* src = c < nq ? q + c * S : k + (c - nq) * S;
    if constexpr (VEC) ld8(src, f);
    else f[0] = ld1(src);
  };
  for (int c = tid; c < n; c += 256) {
    float f[S], ss = 0.f;
    load(c, f);
#pragma unroll
    for (int j = 0; j < S; ++j) {
      ss += f[j] * f[j];
      if (c == tid) first[j] = f[j];
    }
    if (c < nq) sq += ss;
    else sk += ss;
  }
  const bool live = lat_keys(a, row) > 0;  // uniform over the workgroup
  const int p = a.pos[row];
  T* dst = nullptr;
  if (live) {
    dst = static_cast<T*>(a.cache) +
          ((size_t)lat_page(a, a.slot[row], p / LAT_PAGE) * LAT_PAGE + p % LAT_PAGE) * (a.krp + a.rp);
    for (int c = tid; c < a.rp; c += 256) st1(dst + a.krp + c, c < a.rot_dim ? lat_rot(a, k + a.kv_rank, c, p) : 0.f);
  }
  block_sum2(sq, sk, part);
  const float rq = 1.f / sqrtf(sq / (float)a.q_rank + a.eps), rk = 1.f / sqrtf(sk / (float)a.kv_rank + a.eps);
  for (int c = tid; c < n; c += 256) {
    float f[S];
    if (c == tid) {
#pragma unroll
      for (int j = 0; j < S; ++j) f[j] = first[j];
    } else {
      load(c, f);
    }
    const bool isq = c < nq;
    const int o = (isq ? c : c - nq) * S;
    const float* g = (isq ? gq : gk) + o;
    const float r = isq ? rq : rk;
#pragma unroll
    for (int j = 0; j < S; ++j) f[j] *= r * g[j];
    if (!isq && !live) continue;
    T* d = isq ? cq + (size_t)row * ldc + o : dst + o;
    if constexpr (VEC) st8(d, f);
    else st1(d, f[0]);
  }
  if (live)
    for (int c = a.kv_rank + tid; c < a.krp; c += 256) st1(dst + c, 0.f);
}

// wk: [heads][dkp][krp] (row d = the key's dimension d); qt: [entries][heads][krp + rp]
template <typename T>
__global__ __launch_bounds__(256) void absorb_kernel(LatentArgs a, const T* __restrict__ q, int ldq,
                                                     const T* __restrict__ wk, T* __restrict__ qt) {
  const int e = blockIdx.x, h = blockIdx.y, row = a.index ? a.index[e] : e;
  const T* qh = q + (size_t)row * ldq + (size_t)h * (a.dkp + a.rp);
  T* o = qt + ((size_t)e * a.heads + h) * (a.krp + a.rp);
  const T* w = wk + (size_t)h * a.dkp * a.krp;
  for (int j = threadIdx.x; j < a.krp; j += 256) {
    float s = 0.f;
    for (int d = 0; d < a.dim; ++d) s += ld1(qh + d) * ld1(w + (size_t)d * a.krp + j);
    st1(o + j, s);
  }
  const bool live = lat_keys(a, row) > 0;
  for (int j = threadIdx.x; j < a.rp; j += 256)
    st1(o + a.krp + j, live && j < a.rot_dim ? lat_rot(a, qh + a.dkp, j, a.pos[row]) : 0.f);
}

// po: [entries][heads][ns][krp] unnormalised sums, pm: [entries][heads][ns][2] (max in log2 units, sum)
template <typename T>
__global__ __launch_bounds__(256) void attend_kernel(LatentArgs a, const T* __restrict__ qt, int ns,
                                                     float* __restrict__ po, float* __restrict__ pm) {
  extern __shared__ float sm[];  // [krp + rp] query, [krp] running sums, [256] weights, [4]
  const int cw = a.krp + a.rp, tid = threadIdx.x;
  float* sq = sm;
  float* so = sm + cw;
  float* sp = so + a.krp;
  float* part = sp + 256;
  const int e = blockIdx.x, h = blockIdx.y, s = blockIdx.z, row = a.index ? a.index[e] : e;
  const size_t out = ((size_t)e * a.heads + h) * ns + s;
  const int len = lat_keys(a, row), nb = (len + LAT_PAGE - 1) / LAT_PAGE, slot = a.slot[row];
  const int k0 = nb * s / ns * LAT_PAGE, k1 = min(len, nb * (s + 1) / ns * LAT_PAGE);
  const T* qh = qt + ((size_t)e * a.heads + h) * cw;
  const float sl2 = a.scale * 1.4426950408889634f;
  for (int c = tid; c < cw; c += 256) sq[c] = ld1(qh + c) * sl2;
  for (int c = tid; c < a.krp; c += 256) so[c] = 0.f;
  float m = -INFINITY, l = 0.f;
  const T* cache = static_cast<const T*>(a.cache);
  for (int kb = k0; kb < k1; kb += 256) {
    __syncthreads();
    const int key = kb + tid;
    float sc = -INFINITY;
    if (key < k1) {
      const T* c = cache + ((size_t)lat_page(a, slot, key / LAT_PAGE) * LAT_PAGE + key % LAT_PAGE) * cw;
      sc = 0.f;
      for (int d = 0; d < cw; ++d) sc += sq[d] * ld1(c + d);
    }
    const float mn = fmaxf(m, block_max(sc, part));
    const float alpha = __builtin_amdgcn_exp2f(m - mn);
    const float p = key < k1 ? __builtin_amdgcn_exp2f(sc - mn) : 0.f;
    sp[tid] = p;
    l = l * alpha + block_sum(p, part);  // its barriers also publish sp
    m = mn;
    const int nk = min(256, k1 - kb);
    for (int d = tid; d < a.krp; d += 256) {
      float o = so[d] * alpha;
      for (int j = 0; j < nk; ++j) {
        const int kj = kb + j;
        o += sp[j] * ld1(cache + ((size_t)lat_page(a, slot, kj / LAT_PAGE) * LAT_PAGE + kj % LAT_PAGE) * cw + d);
      }
      so[d] = o;
    }
  }
  __syncthreads();
  for (int d = tid; d < a.krp; d += 256) po[out * a.krp + d] = so[d];
  if (tid == 0) {
    pm[out * 2] = m;
    pm[out * 2 + 1] = l;
  }
}

// wv: [heads][krp][dvp]; out row: [heads][dvp] at row, gate (optional) at column og of its row
template <typename T>
__global__ __launch_bounds__(256) void value_kernel(LatentArgs a, const float* __restrict__ po,
                                                    const float* __restrict__ pm, int ns, const T* __restrict__ wv,
                                                    const T* __restrict__ gate, int ldg, T* __restrict__ out, int ldo) {
  extern __shared__ float so[];  // [krp]
  const int e = blockIdx.x, h = blockIdx.y, row = a.index ? a.index[e] : e;
  const size_t b = ((size_t)e * a.heads + h) * ns;
  float M = -INFINITY, L = 0.f;
  for (int s = 0; s < ns; ++s) M = fmaxf(M, pm[(b + s) * 2]);
  if (M == -INFINITY) M = 0.f;
  for (int s = 0; s < ns; ++s) L += pm[(b + s) * 2 + 1] * __builtin_amdgcn_exp2f(pm[(b + s) * 2] - M);
  const float inv = L > 0.f ? 1.f / L : 0.f;
  for (int d = threadIdx.x; d < a.krp; d += 256) {
    float o = 0.f;
    for (int s = 0; s < ns; ++s) o += po[(b + s) * a.krp + d] * __builtin_amdgcn_exp2f(pm[(b + s) * 2] - M);
    so[d] = o * inv;
  }
  __syncthreads();
  const T* w = wv + (size_t)h * a.krp * a.dvp;
  for (int j = threadIdx.x; j < a.dvp; j += 256) {
    float v = 0.f;
    for (int d = 0; d < a.kv_rank; ++d) v += so[d] * ld1(w + (size_t)d * a.dvp + j);
    if (gate) v *= sigmoid(ld1(gate + (size_t)row * ldg + (size_t)h * a.dvp + j));
    st1(out + (size_t)row * ldo + (size_t)h * a.dvp + j, v);
  }
}

// one wave per cached token, four per workgroup; src: (slot, position) of token t
__global__ __launch_bounds__(256) void gather_kernel(LatentArgs a, const int* __restrict__ src, int n,
                                                     bf16_raw* __restrict__ out) {
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63, cw = a.krp + a.rp;
  if (t >= n) return;
  const int slot = src[2 * t], p = src[2 * t + 1];
  const bf16_raw* c = static_cast<const bf16_raw*>(a.cache) +
                      ((size_t)lat_page(a, slot, p / LAT_PAGE) * LAT_PAGE + p % LAT_PAGE) * cw;
  for (int j = lane; j < cw / 8; j += 64) st16(out + (size_t)t * cw + j * 8, ld16(c + j * 8));
}

bool args_ok(const LatentArgs* a, int n) {
  return a && n >= 1 && a->cache && a->table && a->slot && a->pos && a->max_pages >= 1 && a->n_pages >= 1 && a->heads >= 1 &&
         a->dim >= 1 && a->dim <= a->dkp && a->rot_dim >= 2 && a->rot_dim <= a->rp && a->rot_dims >= 2 &&
         a->rot_dims % 2 == 0 && a->rot_dims <= a->rot_dim && a->vdim >= 1 && a->vdim <= a->dvp && a->kv_rank >= 1 &&
         a->kv_rank <= a->krp && a->q_rank >= 1 && a->cos_t && a->sin_t && a->dkp % 64 == 0 && a->rp % 64 == 0 &&
         a->dvp % 64 == 0 && a->krp % 64 == 0;
}

}  // namespace

extern "C" int lsa_latent_append(int f32, const LatentArgs* a, int rows, const void* in, int ldi, int oq, int ok,
                                 const float* gq, const float* gk, void* cq, int ldc, hipStream_t s) {
  if (!args_ok(a, rows) || a->index || oq < 0 || ok < 0 || ldi < oq + a->q_rank || ldi < ok + a->kv_rank + a->rot_dim ||
      ldc < a->q_rank)
    return LSA_BAD_SHAPE;
  const bool vec = !f32 && !((a->q_rank | a->kv_rank | oq | ok | ldi | ldc) % 8) && !(((uintptr_t)in | (uintptr_t)cq) % 16);
  if (f32)
    append_kernel<float, false><<<rows, 256, 0, s>>>(*a, (const float*)in, ldi, oq, ok, gq, gk, (float*)cq, ldc);
  else if (vec)
    append_kernel<bf16_raw, true><<<rows, 256, 0, s>>>(*a, (const bf16_raw*)in, ldi, oq, ok, gq, gk, (bf16_raw*)cq, ldc);
  else
    append_kernel<bf16_raw, false><<<rows, 256, 0, s>>>(*a, (const bf16_raw*)in, ldi, oq, ok, gq, gk, (bf16_raw*)cq, ldc);
  LSA_CHECK_LAUNCH();
  return LSA_OK;
}

extern "C" int lsa_latent_absorb(int f32, const LatentArgs* a, int n, const void* q, int ldq, const void* wk, void* qt,
                                 hipStream_t s) {
  if (!args_ok(a, n) || ldq < a->heads * (a->dkp + a->rp)) return LSA_BAD_SHAPE;
  dim3 grid(n, a->heads);
  if (f32) absorb_kernel<float><<<grid, 256, 0, s>>>(*a, (const float*)q, ldq, (const float*)wk, (float*)qt);
  else absorb_kernel<bf16_raw><<<grid, 256, 0, s>>>(*a, (const bf16_raw*)q, ldq, (const bf16_raw*)wk, (bf16_raw*)qt);
  LSA_CHECK_LAUNCH();
  return LSA_OK;
}

extern "C" int lsa_latent_attend(int f32, const LatentArgs* a, int n, const void* qt, int ns, float* po, float* pm,
                                 hipStream_t s) {
  if (!args_ok(a, n) || ns < 1 || ns > 64) return LSA_BAD_SHAPE;
  const size_t lds = (size_t)(2 * a->krp + a->rp + 256 + 4) * 4;
  if (lds > 64 * 1024) return LSA_UNSUPPORTED;
  dim3 grid(n, a->heads, ns);
  if (f32) attend_kernel<float><<<grid, 256, lds, s>>>(*a, (const float*)qt, ns, po, pm);
  else attend_kernel<bf16_raw><<<grid, 256, lds, s>>>(*a, (const bf16_raw*)qt, ns, po, pm);
  LSA_CHECK_LAUNCH();
  return LSA_OK;
}

extern "C" int lsa_latent_value(int f32, const LatentArgs* a, int n, const float* po, const float* pm, int ns,
                                const void* wv, const void* gate, int ldg, void* out, int ldo, hipStream_t s) {
  if (!args_ok(a, n) || ns < 1 || ns > 64 || ldo < a->heads * a->dvp) return LSA_BAD_SHAPE;
  const size_t lds = (size_t)a->krp * 4;
  if (lds > 64 * 1024) return LSA_UNSUPPORTED;
  dim3 grid(n, a->heads);
  if (f32)
    value_kernel<float><<<grid, 256, lds, s>>>(*a, po, pm, ns, (const float*)wv, (const float*)gate, ldg, (float*)out, ldo);
  else
    value_kernel<bf16_raw><<<grid, 256, lds, s>>>(*a, po, pm, ns, (const bf16_raw*)wv, (const bf16_raw*)gate, ldg,
                                                 (bf16_raw*)out, ldo);
  LSA_CHECK_LAUNCH();
  return LSA_OK;
}

extern "C" int lsa_latent_gather(const LatentArgs* a, const int* src, int n, void* out, hipStream_t s) {
  if (!args_ok(a, n) || !src || !out) return LSA_BAD_SHAPE;
  gather_kernel<<<(n + 3) / 4, 256, 0, s>>>(*a, src, n, (bf16_raw*)out);
  LSA_CHECK_LAUNCH();
  return LSA_OK;
}
