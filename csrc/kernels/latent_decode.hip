// Latent attention in the absorbed form on MFMA (latent.h): decode rows and short portions, bf16.
//
//   lsa_latent_absorb_mfma  q~^T[latent][row] = W_uk^h^T . q_h^T per head; rotated part behind it
//   lsa_latent_attend_mfma  one workgroup per (row, group of HT x 16 heads, split): every cached
//       entry is read from memory ONCE for all heads of the group and once from LDS per use:
//       * a 64-token page arrives by LDS-DMA into a double buffer (the next page is in flight
//         while this one is computed), chunk-swizzled on the source address
//       * S^T[key][head] = C . q~^T: a wave takes 16 keys and all or half of the head tiles (A = page
//         rows by ds_read_b128, B = its queries, in registers for the whole launch)
//       * softmax: column maxima meet in LDS, every lane then works on its own keys in fp32
//       * O^T[latent][head] += C^T . P^T: the waves take equal parts of the latent, C^T by the
//         hardware-transposed LDS read of the same page image, P^T (bf16) through LDS
//   lsa_latent_value_mfma   merge of the splits, then W_uv^h per head, output gate in the epilogue
#include "latent.h"

namespace {

typedef short v4s_t __attribute__((ext_vector_type(4)));

// chunk swizzle of row r in a page image of NCH 16-B chunks per row: both the 16-lane ds_read_b128
// groups (rows l16) and the transposed reads hit distinct bank slots. NCH = 8 (mod 16): odd rows
// start half a bank row later, so (r >> 1) & 7 completes the sixteen slots.
template <int NCH>
LSA_DEVICE int swz(int r) {
  if constexpr (NCH % 16 == 0) return ((r & 3) << 2) ^ (((r >> 2) & 3) << 1);
  else return (r >> 1) & 7;
}

LSA_DEVICE void glds16(const void* src, unsigned char* lds_base) {
  __builtin_amdgcn_global_load_lds(src, (__attribute__((address_space(3))) void*)lds_base, 16, 0, 0);
}

constexpr int RP = 64;   // rotated part of a cache entry

// Workgroup barrier for LDS traffic alone: the page DMA in flight stays in flight (a fence of
// __syncthreads would drain it).
LSA_DEVICE void lds_barrier() {
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");
}

// waves: four key groups, and with two or more head tiles two head groups in the score step
template <int KRP, int HT>
constexpr int attend_waves() { return HT >= 2 && KRP >= 128 ? 8 : 4; }

template <int KRP, int HT>
__global__ __launch_bounds__((attend_waves<KRP, HT>() * 64), (attend_waves<KRP, HT>() / 4)) void attend_mfma_kernel(
    LatentArgs a, const bf16_raw* __restrict__ qt, int ns, float* __restrict__ po, float* __restrict__ pm) {
  constexpr int NW = attend_waves<KRP, HT>(), HG = NW / 4, QT = HT / HG;  // QT: head tiles per wave's scores
  constexpr int CW = KRP + RP, NCH = CW / 8, KF = CW / 32, DTW = KRP / 16 / NW;
  constexpr int BLK = LAT_PAGE * CW * 2, PPW = BLK / 1024 / NW, C1 = HT * 16;
  static_assert(PPW * NW * 1024 == BLK && DTW >= 1 && QT * HG == HT, "geometry");
  // ONE array: with several, the compiler tells their accesses apart and drains the page DMA before
  // the first read of the other page
  __shared__ __attribute__((aligned(16))) unsigned char smem[2 * BLK + HT * 2 * 64 * 16 + 4 * HT * 16 * 4];
  unsigned char* spt = smem + 2 * BLK;                                       // P^T fragments
  float* smax = reinterpret_cast<float*>(smem + 2 * BLK + HT * 2 * 64 * 16);  // [4 key groups][HT * 16]

  const int e = blockIdx.x, h0 = blockIdx.y * (HT * 16), sp = blockIdx.z;
  const int row = a.index ? a.index[e] : e;
  const int tid = threadIdx.x, lane = tid & 63, g = lane >> 4, l16 = lane & 15;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6), kg = w & 3, t0 = (w >> 2) * QT;
  const int slot = __builtin_amdgcn_readfirstlane(a.slot[row]);
  const int len = __builtin_amdgcn_readfirstlane(lat_keys(a, row));
  const int first = lat_first(a, len), fb = first / LAT_PAGE, nb = (len + LAT_PAGE - 1) / LAT_PAGE - fb;
  const int b0 = fb + nb * sp / ns, b1 = fb + nb * (sp + 1) / ns;
  const bf16_raw* cache = static_cast<const bf16_raw*>(a.cache);
  const float sl2 = a.scale * 1.4426950408889634f;

  auto stage = [&](int page, int buf) {
    const bf16_raw* src = cache + (size_t)page * LAT_PAGE * CW;
#pragma unroll
    for (int s = 0; s < PPW; ++s) {
      const int pc = w * PPW + s, lin = pc * 64 + lane, r = lin / NCH, c = lin % NCH;
      glds16(src + (size_t)r * CW + (c ^ swz<NCH>(r)) * 8, smem + buf * BLK + pc * 1024);
    }
  };
  // lane i holds the page of block pb + i: no memory access (whose wait would drain the DMA) in the loop
  int pb = b0;
  int pages = b0 + lane < b1 ? lat_page(a, slot, b0 + lane) : 0;
  if (b0 < b1) stage(__builtin_amdgcn_readlane(pages, 0), 0);

  u32x4_t qf[QT][KF];
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    const int h = h0 + (t0 + t) * 16 + l16;
    const bf16_raw* q = qt + ((size_t)e * a.heads + min(h, a.heads - 1)) * CW;  // surplus columns are not stored
#pragma unroll
    for (int kf = 0; kf < KF; ++kf) qf[t][kf] = ld16(q + kf * 32 + g * 8);
  }
  // the queries have arrived here, not at their first use inside the loop (whose wait would also
  // drain the next page's DMA, every time around)
#pragma unroll
  for (int t = 0; t < QT; ++t)
#pragma unroll
    for (int kf = 0; kf < KF; ++kf) asm volatile("" : "+v"(qf[t][kf]));

  f32x4_t o[HT][DTW];
  float m_run[HT], l_run[QT];
#pragma unroll
  for (int t = 0; t < HT; ++t) {
    m_run[t] = -INFINITY;
    if (t < QT) l_run[t] = 0.f;
#pragma unroll
    for (int d = 0; d < DTW; ++d) o[t][d] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  }
  // per-lane offsets into a page image: key row 16 kg + l16 (its swizzle depends on l16 alone), and
  // the transposed reads' row 4 g + l16 / 4 (+ 16, + 32: same swizzle)
  const int krow = (kg * 16 + l16) * (CW * 2), ksw = swz<NCH>(l16);
  const int vlo = 4 * g + (l16 >> 2), vrow = vlo * (CW * 2), vsw = swz<NCH>(vlo);

  for (int b = b0; b < b1; ++b) {
    const unsigned char* img = smem + ((b - b0) & 1) * BLK;
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");  // this wave's part of page b has landed
    lds_barrier();  // every wave's, and every wave is done with the other buffer and with spt
    if (b + 1 < b1) {
      if (b + 1 - pb == 64) {
        pb += 64;
        pages = pb + lane < b1 ? lat_page(a, slot, pb + lane) : 0;
      }
      stage(__builtin_amdgcn_readlane(pages, b + 1 - pb), (b + 1 - b0) & 1);
    }

    f32x4_t s[QT], s2[QT];
#pragma unroll
    for (int t = 0; t < QT; ++t) s[t] = s2[t] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int kf = 0; kf < KF; ++kf) {
      const u32x4_t k = *reinterpret_cast<const u32x4_t*>(img + krow + (((kf * 4 + g) ^ ksw) << 4));
#pragma unroll
      for (int t = 0; t < QT; ++t) {
        if (QT <= 2 && (kf & 1)) s2[t] = mfma16(k, qf[t][kf], s2[t]);  // two chains where one would stall
        else s[t] = mfma16(k, qf[t][kf], s[t]);
      }
    }
    // four reads ahead of the MFMAs
    __builtin_amdgcn_sched_group_barrier(0x100, KF < 4 ? KF : 4, 0);
#pragma unroll
    for (int kf = 4; kf < KF; ++kf) {
      __builtin_amdgcn_sched_group_barrier(0x008, QT, 0);
      __builtin_amdgcn_sched_group_barrier(0x100, 1, 0);
    }
    __builtin_amdgcn_sched_group_barrier(0x008, QT * (KF < 4 ? KF : 4), 0);
#pragma unroll
    for (int t = 0; t < QT; ++t) {
      float mx = -INFINITY;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int key = b * LAT_PAGE + kg * 16 + g * 4 + r;
        const float v = key < len && key >= first ? (s[t][r] + s2[t][r]) * sl2 : -INFINITY;
        s[t][r] = v;
        mx = fmaxf(mx, v);
      }
      mx = fmaxf(mx, lane_xor<16>(mx));
      mx = fmaxf(mx, lane_xor<32>(mx));
      if (g == 0) smax[kg * C1 + (t0 + t) * 16 + l16] = mx;
    }
    lds_barrier();
    float mn[HT];
#pragma unroll
    for (int t = 0; t < HT; ++t) {
      const int c = t * 16 + l16;
      // page b holds at least one visible key, so the new maximum is finite
      mn[t] = fmaxf(m_run[t], fmaxf(fmaxf(smax[c], smax[C1 + c]), fmaxf(smax[2 * C1 + c], smax[3 * C1 + c])));
    }
#pragma unroll
    for (int t = 0; t < QT; ++t) {
      const int ta = t0 + t;
      float mt = mn[t], mo = m_run[t];
      if (HG == 2) {  // this wave's head group (wave-uniform)
        mt = t0 ? mn[HT - QT + t] : mt;
        mo = t0 ? m_run[HT - QT + t] : mo;
      }
      float ps = 0.f;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        s[t][r] = __builtin_amdgcn_exp2f(s[t][r] - mt);
        ps += s[t][r];
      }
      l_run[t] = l_run[t] * __builtin_amdgcn_exp2f(mo - mt) + ps;  // this lane's keys; summed at the end
      // fragment f2 = kg / 2 of the 32-key PV step, this wave's half of its eight keys per lane
      st4(reinterpret_cast<bf16_raw*>(spt + (((ta * 2 + (kg >> 1)) * 64 + lane) << 4) + ((kg & 1) << 3)), s[t]);
    }
#pragma unroll
    for (int t = 0; t < HT; ++t) {
      if (__builtin_amdgcn_ballot_w64(mn[t] != m_run[t])) {
        const float alpha = __builtin_amdgcn_exp2f(m_run[t] - mn[t]);
#pragma unroll
        for (int d = 0; d < DTW; ++d) o[t][d] *= alpha;
      }
      m_run[t] = mn[t];
    }
    lds_barrier();
#pragma unroll
    for (int f2 = 0; f2 < 2; ++f2) {
      u32x4_t p[HT];
#pragma unroll
      for (int t = 0; t < HT; ++t) p[t] = *reinterpret_cast<const u32x4_t*>(spt + (((t * 2 + f2) * 64 + lane) << 4));
#pragma unroll
      for (int d = 0; d < DTW; ++d) {
        const int dt = w * DTW + d;
        const unsigned char* v = img + f2 * 32 * (CW * 2) + vrow + (((2 * dt + ((l16 & 3) >> 1)) ^ vsw) << 4) + 8 * (l16 & 1);
        const v4s_t lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) v4s_t*)v);
        const v4s_t hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
            (__attribute__((address_space(3))) v4s_t*)(v + 16 * (CW * 2)));
        u32x4_t c;
        c[0] = __builtin_bit_cast(u32x2_t, lo)[0];
        c[1] = __builtin_bit_cast(u32x2_t, lo)[1];
        c[2] = __builtin_bit_cast(u32x2_t, hi)[0];
        c[3] = __builtin_bit_cast(u32x2_t, hi)[1];
#pragma unroll
        for (int t = 0; t < HT; ++t) o[t][d] = mfma16(c, p[t], o[t][d]);
      }
    }
    // both P fragments and the first latent tiles are read ahead of the MFMAs
    __builtin_amdgcn_sched_group_barrier(0x100, 2 * HT + 4, 0);
#pragma unroll
    for (int i = 2; i < 2 * DTW; ++i) {
      __builtin_amdgcn_sched_group_barrier(0x008, HT, 0);
      __builtin_amdgcn_sched_group_barrier(0x100, 2, 0);
    }
    __builtin_amdgcn_sched_group_barrier(0x008, 2 * HT, 0);
  }

  lds_barrier();  // the last page's maxima have been read
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    l_run[t] += lane_xor<16>(l_run[t]);
    l_run[t] += lane_xor<32>(l_run[t]);
    if (g == 0) smax[kg * C1 + (t0 + t) * 16 + l16] = l_run[t];
  }
  lds_barrier();
#pragma unroll
  for (int t = 0; t < HT; ++t) {
    const int h = h0 + t * 16 + l16;
    if (h >= a.heads) continue;
    const size_t out = ((size_t)e * a.heads + h) * ns + sp;
#pragma unroll
    for (int d = 0; d < DTW; ++d)
      *reinterpret_cast<f32x4_t*>(po + out * KRP + (w * DTW + d) * 16 + 4 * g) = o[t][d];
    if (w == 0 && g == 0) {
      const int c = t * 16 + l16;
      pm[out * 2] = m_run[t];
      pm[out * 2 + 1] = smax[c] + smax[C1 + c] + smax[2 * C1 + c] + smax[3 * C1 + c];
    }
  }
}

// wk: per head the packed [krp][dkp] matrix (common.h fragment order). Grid (16-entry tiles, heads,
// 16-tile stretches of the latent + 1): every wave up to 4 latent tiles; the last z turns the
// rotated parts beside them.
__global__ __launch_bounds__(256) void absorb_mfma_kernel(LatentArgs a, int n, const bf16_raw* __restrict__ q, int ldq,
                                                          const bf16_raw* __restrict__ wk, bf16_raw* __restrict__ qt) {
  const int h = blockIdx.y, e0 = blockIdx.x * 16;
  const int tid = threadIdx.x, lane = tid & 63, g = lane >> 4, l16 = lane & 15, w = tid >> 6;
  const int kf_n = a.dkp / 32, nt_n = a.krp / 16, cw = a.krp + a.rp;
  if (blockIdx.z == gridDim.z - 1) {
    for (int i = tid; i < 16 * a.rp; i += 256) {
      const int ee = e0 + i / a.rp, j = i % a.rp;
      if (ee >= n) break;
      const int rr = a.index ? a.index[ee] : ee;
      const bf16_raw* qr = q + (size_t)rr * ldq + (size_t)h * (a.dkp + a.rp) + a.dkp;
      const int p = a.pos[rr];
      const bool live = j < a.rot_dim && p >= 0 && p < a.max_pages * LAT_PAGE;
      st1(qt + ((size_t)ee * a.heads + h) * cw + a.krp + j, live ? lat_rot(a, qr, j, p) : 0.f);
    }
    return;
  }
  const int e = min(e0 + l16, n - 1);  // surplus columns repeat the last entry and are not stored
  const int row = a.index ? a.index[e] : e;
  const bf16_raw* qh = q + (size_t)row * ldq + (size_t)h * (a.dkp + a.rp);
  const int t0 = blockIdx.z * 16 + w * 4;
  if (t0 >= nt_n) return;  // krp % 64 == 0: whole groups of four tiles
  const bf16_raw* wh = wk + ((size_t)h * nt_n + t0) * kf_n * 512 + lane * 8;
  f32x4_t acc[4];
#pragma unroll
  for (int t = 0; t < 4; ++t) acc[t] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < kf_n; k0 += 2) {  // dkp % 64 == 0
    u32x4_t wt[2][4], b[2];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
#pragma unroll
      for (int t = 0; t < 4; ++t) wt[u][t] = ld16(wh + ((size_t)t * kf_n + k0 + u) * 512);
      b[u] = ld16(qh + (k0 + u) * 32 + g * 8);
    }
#pragma unroll
    for (int u = 0; u < 2; ++u)
#pragma unroll
      for (int t = 0; t < 4; ++t) acc[t] = mfma16(wt[u][t], b[u], acc[t]);
  }
  if (e0 + l16 < n) {
    bf16_raw* o = qt + ((size_t)e * a.heads + h) * cw;
#pragma unroll
    for (int t = 0; t < 4; ++t) st4(o + (t0 + t) * 16 + 4 * g, acc[t]);
  }
}

// wv: per head the packed [dvp][krp] matrix. Grid (16-entry tiles, heads, 8-tile stretches of the
// value); eight waves, one 16-wide value tile each, whose weights are requested before the merge.
template <int KRP>
__global__ __launch_bounds__(512) void value_mfma_kernel(LatentArgs a, int n, const float* __restrict__ po,
                                                         const float* __restrict__ pm, int ns,
                                                         const bf16_raw* __restrict__ wv, const bf16_raw* __restrict__ gate,
                                                         int ldg, bf16_raw* __restrict__ out, int ldo) {
  constexpr int KF = KRP / 32, LD = KRP + 8;
  __shared__ __attribute__((aligned(16))) bf16_raw so[16 * LD];
  __shared__ float wgt[16][64];
  const int h = blockIdx.y, e0 = blockIdx.x * 16;
  const int tid = threadIdx.x, lane = tid & 63, g = lane >> 4, l16 = lane & 15, w = tid >> 6;
  const int t = blockIdx.z * 8 + w;
  const bool work = t * 16 < a.dvp;
  u32x4_t wf[KF];
  {
    const bf16_raw* wh = wv + ((size_t)h * (a.dvp / 16) + (work ? t : 0)) * KF * 512 + lane * 8;
#pragma unroll
    for (int kf = 0; kf < KF; ++kf) wf[kf] = ld16(wh + (size_t)kf * 512);
  }
  if (ns > 1) {  // weights of the splits (ns <= 64): a wave per entry, a lane per split
    for (int r = w; r < 16 && e0 + r < n; r += 8) {
      const float* p = pm + ((size_t)(e0 + r) * a.heads + h) * ns * 2;
      const float m = lane < ns ? p[2 * lane] : -INFINITY, l = lane < ns ? p[2 * lane + 1] : 0.f;
      float M = wave_max(m);
      if (M == -INFINITY) M = 0.f;
      const float f = __builtin_amdgcn_exp2f(m - M), L = wave_sum(l * f) + lat_sink(a, h, M);
      wgt[r][lane] = L > 0.f ? f / L : 0.f;
    }
  }
  __syncthreads();
  for (int i = tid; i < 16 * (KRP / 4); i += 512) {
    const int r = i / (KRP / 4), c = (i % (KRP / 4)) * 4, e = e0 + r;
    f32x4_t v = f32x4_t{0.f, 0.f, 0.f, 0.f};
    if (e < n) {
      const size_t b = ((size_t)e * a.heads + h) * ns;
      const float* p = po + b * KRP + c;
      if (ns == 1) {
        const float m = pm[b * 2], L = pm[b * 2 + 1] + (m == -INFINITY ? 0.f : lat_sink(a, h, m));
        v = *reinterpret_cast<const f32x4_t*>(p) * (L > 0.f ? 1.f / L : 0.f);
      } else {
        int s = 0;
        for (; s < ns; s += 8) {  // eight reads in flight (past the last split: its value again, times 0)
          f32x4_t x[8];
#pragma unroll
          for (int u = 0; u < 8; ++u) x[u] = *reinterpret_cast<const f32x4_t*>(p + (size_t)min(s + u, ns - 1) * KRP);
#pragma unroll
          for (int u = 0; u < 8; ++u) v += x[u] * (s + u < ns ? wgt[r][s + u] : 0.f);
        }
      }
    }
    st4(so + r * LD + c, v);
  }
  __syncthreads();
  const int e = e0 + l16;
  f32x4_t acc = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int kf = 0; kf < KF; ++kf) acc = mfma16(wf[kf], ld16(so + l16 * LD + kf * 32 + g * 8), acc);
  if (!work || e >= n) return;
  const int row = a.index ? a.index[e] : e, col = h * a.dvp + t * 16 + 4 * g;
  if (gate) {
    const u32x2_t gb = *reinterpret_cast<const u32x2_t*>(gate + (size_t)row * ldg + col);
    acc[0] *= sigmoid(__uint_as_float(gb[0] << 16));
    acc[1] *= sigmoid(__uint_as_float(gb[0] & 0xffff0000u));
    acc[2] *= sigmoid(__uint_as_float(gb[1] << 16));
    acc[3] *= sigmoid(__uint_as_float(gb[1] & 0xffff0000u));
  }
  st4(out + (size_t)row * ldo + col, acc);
}

bool size_ok(const LatentArgs* a, int n) {
  return a && n >= 1 && a->window >= 0 && a->cache && a->table && a->slot && a->pos && a->max_pages >= 1 && a->n_pages >= 1 && a->heads >= 1 &&
         a->dim >= 1 && a->dim <= a->dkp && a->dkp % 64 == 0 && a->rp == RP && a->rot_dim >= 2 && a->rot_dim <= RP &&
         a->rot_dims >= 2 && a->rot_dims % 2 == 0 && a->rot_dims <= a->rot_dim && a->vdim >= 1 && a->vdim <= a->dvp &&
         a->dvp % 64 == 0 && a->kv_rank >= 1 && a->kv_rank <= a->krp && a->cos_t && a->sin_t &&
         (a->krp == 64 || a->krp == 128 || a->krp == 256 || a->krp == 512);
}

}  // namespace

extern "C" int lsa_latent_absorb_mfma(const LatentArgs* a, int n, const void* q, int ldq, const void* wk, void* qt,
                                      hipStream_t s) {
  if (!size_ok(a, n) || ldq < a->heads * (a->dkp + a->rp) || ldq % 8 || (uintptr_t)q % 16 || (uintptr_t)qt % 16)
    return LSA_BAD_SHAPE;
  dim3 grid((n + 15) / 16, a->heads, (a->krp / 16 + 15) / 16 + 1);
  absorb_mfma_kernel<<<grid, 256, 0, s>>>(*a, n, (const bf16_raw*)q, ldq, (const bf16_raw*)wk, (bf16_raw*)qt);
  LSA_CHECK_LAUNCH();
  return LSA_OK;
}

extern "C" int lsa_latent_attend_mfma(const LatentArgs* a, int n, const void* qt, int ns, float* po, float* pm,
                                      hipStream_t s) {
  if (!size_ok(a, n) || ns < 1 || ns > 64 || (uintptr_t)qt % 16 || (uintptr_t)po % 16) return LSA_BAD_SHAPE;
  // head tiles per workgroup; four tiles of 512-wide latents do not fit the register file
  const int tiles = (a->heads + 15) / 16, ht = tiles >= 3 ? (a->krp == 512 ? 2 : 4) : tiles;
  dim3 grid(n, (tiles + ht - 1) / ht, ns);
#define LSA_A(K, T) attend_mfma_kernel<K, T><<<grid, (attend_waves<K, T>() * 64), 0, s>>>(*a, (const bf16_raw*)qt, ns, po, pm)
#define LSA_K(K)                                 \
  if (ht == 1) LSA_A(K, 1);                      \
  else if (ht == 2) LSA_A(K, 2);                 \
  else if constexpr (K < 512) LSA_A(K, 4);
  switch (a->krp) {
    case 64: LSA_K(64) break;
    case 128: LSA_K(128) break;
    case 256: LSA_K(256) break;
    case 512: LSA_K(512) break;
    default: return LSA_UNSUPPORTED;
  }
#undef LSA_K
#undef LSA_A
  LSA_CHECK_LAUNCH();
  return LSA_OK;
}

extern "C" int lsa_latent_value_mfma(const LatentArgs* a, int n, const float* po, const float* pm, int ns, const void* wv,
                                     const void* gate, int ldg, void* out, int ldo, hipStream_t s) {
  if (!size_ok(a, n) || ns < 1 || ns > 64 || ldo < a->heads * a->dvp || ldo % 4 || (uintptr_t)out % 8 || (uintptr_t)po % 16)
    return LSA_BAD_SHAPE;
  if (gate && (ldg % 4 || (uintptr_t)gate % 8)) return LSA_BAD_SHAPE;
  dim3 grid((n + 15) / 16, a->heads, (a->dvp + 127) / 128);
#define LSA_V(K)                                                                                                       \
  case K:                                                                                                              \
    value_mfma_kernel<K><<<grid, 512, 0, s>>>(*a, n, po, pm, ns, (const bf16_raw*)wv, (const bf16_raw*)gate, ldg,      \
                                              (bf16_raw*)out, ldo);                                                    \
    break;
  switch (a->krp) {
    LSA_V(64) LSA_V(128) LSA_V(256) LSA_V(512)
    default: return LSA_UNSUPPORTED;
  }
#undef LSA_V
  LSA_CHECK_LAUNCH();
  return LSA_OK;
}
