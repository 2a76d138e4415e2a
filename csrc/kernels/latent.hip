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

// in: row of the fused input projection, query latent at column oq, [key latent | rotated part] at ok
template <typename T>
__global__ __launch_bounds__(256) void append_kernel(LatentArgs a, const T* __restrict__ in, int ldi, int oq, int ok,
                                                     const float* __restrict__ gq, const float* __restrict__ gk,
                                                     T* __restrict__ cq, int ldc) {
  __shared__ float part[2][4];
  const int row = blockIdx.x, tid = threadIdx.x;
  const T* q = in + (size_t)row * ldi + oq;
  const T* k = in + (size_t)row * ldi + ok;
  float sq = 0.f, sk = 0.f;
  for (int c = tid; c < a.q_rank; c += 256) {
    const float v = ld1(q + c);
    sq += v * v;
  }
  for (int c = tid; c < a.kv_rank; c += 256) {
    const float v = ld1(k + c);
    sk += v * v;
  }
  block_sum2(sq, sk, part);
  const float rq = 1.f / sqrtf(sq / (float)a.q_rank + a.eps), rk = 1.f / sqrtf(sk / (float)a.kv_rank + a.eps);
  for (int c = tid; c < a.q_rank; c += 256) st1(cq + (size_t)row * ldc + c, ld1(q + c) * rq * gq[c]);
  if (lat_keys(a, row) == 0) return;  // uniform over the workgroup
  const int p = a.pos[row];
  T* dst = static_cast<T*>(a.cache) +
           ((size_t)lat_page(a, a.slot[row], p / LAT_PAGE) * LAT_PAGE + p % LAT_PAGE) * (a.krp + a.rp);
  for (int c = tid; c < a.krp; c += 256) st1(dst + c, c < a.kv_rank ? ld1(k + c) * rk * gk[c] : 0.f);
  for (int c = tid; c < a.rp; c += 256) st1(dst + a.krp + c, c < a.rot_dim ? lat_rot(a, k + a.kv_rank, c, p) : 0.f);
}

// The same in bf16 with one wave per row (no barrier), both latents in registers: NV stretches of 8
// values per lane (ranks and column offsets multiples of 8, (q_rank + kv_rank) / 8 <= 64 NV).
template <int NV>
__global__ __launch_bounds__(256) void append_wave_kernel(LatentArgs a, int rows, const bf16_raw* __restrict__ in, int ldi,
                                                          int oq, int ok, const float* __restrict__ gq,
                                                          const float* __restrict__ gk, bf16_raw* __restrict__ cq, int ldc) {
  const int row = blockIdx.x * (blockDim.x >> 6) + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (row >= rows) return;
  const bf16_raw* q = in + (size_t)row * ldi + oq;
  const bf16_raw* k = in + (size_t)row * ldi + ok;
  const int nq = a.q_rank / 8, n = nq + a.kv_rank / 8;
  u32x4_t v[NV];
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int c = lane + 64 * j;
    v[j] = c < n ? ld16(c < nq ? q + c * 8 : k + (c - nq) * 8) : u32x4_t{0u, 0u, 0u, 0u};
  }
  const int p = a.pos[row];
  bf16_raw* dst = nullptr;
  if (lat_keys(a, row) > 0) {  // uniform over the wave
    dst = static_cast<bf16_raw*>(a.cache) +
          ((size_t)lat_page(a, a.slot[row], p / LAT_PAGE) * LAT_PAGE + p % LAT_PAGE) * (a.krp + a.rp);
    for (int c = lane; c < a.rp; c += 64) st1(dst + a.krp + c, c < a.rot_dim ? lat_rot(a, k + a.kv_rank, c, p) : 0.f);
    for (int c = a.kv_rank + lane; c < a.krp; c += 64) st1(dst + c, 0.f);
  }
  float sq = 0.f, sk = 0.f;
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    float f[8], s = 0.f;
    unpack8(v[j], f);
#pragma unroll
    for (int i = 0; i < 8; ++i) s += f[i] * f[i];
    if (lane + 64 * j < nq) sq += s;
    else sk += s;
  }
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  const float rq = 1.f / sqrtf(sq / (float)a.q_rank + a.eps), rk = 1.f / sqrtf(sk / (float)a.kv_rank + a.eps);
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int c = lane + 64 * j;
    const bool isq = c < nq;
    if (c >= n || (!isq && !dst)) continue;
    const int o = (isq ? c : c - nq) * 8;
    const float* g = (isq ? gq : gk) + o;
    const f32x4_t g0 = *reinterpret_cast<const f32x4_t*>(g), g1 = *reinterpret_cast<const f32x4_t*>(g + 4);
    const float r = isq ? rq : rk;
    float f[8];
    unpack8(v[j], f);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      f[i] *= r * g0[i];
      f[4 + i] *= r * g1[i];
    }
    st16(isq ? cq + (size_t)row * ldc + o : dst + o, pack8(f));
  }
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
  const int len = lat_keys(a, row), first = lat_first(a, len), slot = a.slot[row];
  const int fb = first / LAT_PAGE, nb = (len + LAT_PAGE - 1) / LAT_PAGE - fb;
  const int k0 = max(first, (fb + nb * s / ns) * LAT_PAGE), k1 = min(len, (fb + nb * (s + 1) / ns) * LAT_PAGE);
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
  L += lat_sink(a, h, M);
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
  return a && n >= 1 && a->window >= 0 && a->cache && a->table && a->slot && a->pos && a->max_pages >= 1 && a->n_pages >= 1 && a->heads >= 1 &&
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
  const int n8 = (a->q_rank + a->kv_rank) / 8;
  const bool wave = !f32 && n8 <= 512 && !((a->q_rank | a->kv_rank | oq | ok | ldi | ldc) % 8) &&
                    !(((uintptr_t)in | (uintptr_t)cq | (uintptr_t)gq | (uintptr_t)gk) % 16);
  const int wpg = rows >= 2048 ? 4 : 1;  // few rows: one to a CU
#define LSA_W(NV)                                                                                                  \
  append_wave_kernel<NV><<<(rows + wpg - 1) / wpg, wpg * 64, 0, s>>>(*a, rows, (const bf16_raw*)in, ldi, oq, ok,  \
                                                                    gq, gk, (bf16_raw*)cq, ldc)
  if (wave && n8 <= 128) LSA_W(2);
  else if (wave && n8 <= 320) LSA_W(5);
  else if (wave) LSA_W(8);
  else if (f32) append_kernel<float><<<rows, 256, 0, s>>>(*a, (const float*)in, ldi, oq, ok, gq, gk, (float*)cq, ldc);
  else append_kernel<bf16_raw><<<rows, 256, 0, s>>>(*a, (const bf16_raw*)in, ldi, oq, ok, gq, gk, (bf16_raw*)cq, ldc);
#undef LSA_W
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
