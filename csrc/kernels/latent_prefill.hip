// Latent attention in the expanded form (latent.h): flash attention of a portion's query tiles over
// keys and values multiplied out of the cached latents, bf16 on MFMA.
//
// The work unit and the pipeline are those of the flash prefill kernel (attn_prefill.hip): one
// query tile of one sequence x one head, eight waves of 16 rows, K and V blocks of 64 keys by
// LDS-DMA into a double buffer, S^T = K . Q^T, per-lane online softmax, O^T += V^T . P^T with P^T
// taken from the S^T accumulators. What differs: a key is two pieces from two places (the head's
// unrotated part beside its value in ``kv``, the rotated part shared by all heads behind the
// gathered latent in ``lat``), key and value have different widths, the query's rotated part is
// turned while it is loaded, and the output gate is applied to the finished tile.
#include "latent.h"

namespace {

constexpr int BKV = 64, NWV = 8, NTHR = NWV * 64, NBUF = 2, RP = 64;

// as PrefillTile: kv0 = first gathered row of the sequence, of position ``base``; kvlen counts from there
struct LatTile {
  int row0, nrows, kv0, pos0, kvlen, base, pad1, pad2;
};

typedef short v4s_t __attribute__((ext_vector_type(4)));

template <int NC>
LSA_DEVICE int swz(int r) {
  if constexpr (NC == 16) return ((r & 3) << 2) ^ (((r >> 2) & 3) << 1);
  else return (r >> 1) & 7;
}
template <int NC>
LSA_DEVICE int sw_off(int r, int ch) {
  return r * (NC * 16) + ((ch ^ swz<NC>(r)) << 4);
}

LSA_DEVICE void glds16(const void* src, unsigned char* lds_base) {
  __builtin_amdgcn_global_load_lds(src, (__attribute__((address_space(3))) void*)lds_base, 16, 0, 0);
}

template <int DK, int DV>
__global__ __launch_bounds__(NTHR, 4) void latent_prefill_kernel(LatentArgs a, const LatTile* __restrict__ tiles,
                                                              const bf16_raw* __restrict__ q, int ldq,
                                                              const bf16_raw* __restrict__ kv, int ldkv,
                                                              const bf16_raw* __restrict__ lat,
                                                              const bf16_raw* __restrict__ gate, int ldg,
                                                              bf16_raw* __restrict__ out, int ldo) {
  constexpr int KD = DK + RP, KF = KD / 32, DT = DV / 16, NCK = KD / 8, NCV = DV / 8;
  constexpr int KBLK = BKV * KD * 2, VBLK = BKV * DV * 2;
  constexpr int KPW = KBLK / 1024 / NWV, VPW = VBLK / 1024 / NWV;  // DMA pieces per wave
  static_assert(KPW * NWV * 1024 == KBLK && VPW * NWV * 1024 == VBLK, "geometry");
  __shared__ __attribute__((aligned(16))) unsigned char smem[NBUF * (KBLK + VBLK)];

  const int H = a.heads, n_tiles = gridDim.x / H;
  int tix, head;
  if (H % 8 == 0) {  // XCD x owns heads x, x + 8, ...: their expanded keys and values stay in its L2
    const int x = blockIdx.x % 8, j = blockIdx.x / 8, hx = H / 8;
    tix = j / hx;
    head = (j % hx) * 8 + x;
  } else {
    tix = blockIdx.x % n_tiles;
    head = blockIdx.x / n_tiles;
  }
  const LatTile tile = tiles[tix];
  const int tid = threadIdx.x, lane = tid & 63, g = lane >> 4, l16 = lane & 15;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int my_row = w * 16 + l16;
  const bool row_ok = my_row < tile.nrows;
  const int rel0 = tile.pos0 - tile.base, my_pos = rel0 + my_row;  // positions among the gathered rows

  u32x4_t qf[KF];
  {
    const bf16_raw* qr = q + (size_t)(tile.row0 + (row_ok ? my_row : 0)) * ldq + (size_t)head * KD;
#pragma unroll
    for (int kf = 0; kf < DK / 32; ++kf) qf[kf] = ld16(qr + kf * 32 + g * 8);
    const int p = tile.pos0 + (row_ok ? my_row : 0);
#pragma unroll
    for (int kf = DK / 32; kf < KF; ++kf) {
      float v[8];
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const int i = kf * 32 + g * 8 + j - DK;
        v[j] = i < a.rot_dim ? lat_rot(a, qr + DK, i, p) : 0.f;
      }
      qf[kf] = pack8(v);
    }
    // the query has arrived here, not at its first use inside the block loop (whose wait would also
    // drain the next block's DMA, every time around)
#pragma unroll
    for (int kf = 0; kf < KF; ++kf) asm volatile("" : "+v"(qf[kf]));
  }
  const int lim = min(rel0 + tile.nrows, tile.kvlen);
  const int my_lim = min(my_pos + 1, tile.kvlen);
  const int wave_lim = min(rel0 + min(w * 16 + 16, tile.nrows), tile.kvlen);
  const int wave_min_lim = min(rel0 + w * 16 + 1, tile.kvlen);
  // first visible key: of this lane's row, of the wave's first and last row, of the tile
  const int win = a.window > 0 ? a.window : 0x3fffffff;
  const int my_first = my_pos + 1 - win, wave_first = rel0 + w * 16 + 1 - win, wave_max_first = wave_first + 15;
  const int kb_first = max(0, rel0 + 1 - win) / BKV;
  const int nkb = (lim + BKV - 1) / BKV;
  const int cw = a.krp + RP;
  const bf16_raw* kvb = kv + (size_t)tile.kv0 * ldkv + (size_t)head * (DK + DV);
  const bf16_raw* rotb = lat + (size_t)tile.kv0 * cw + a.krp;
  const float sl2 = a.scale * 1.4426950408889634f;

  auto stage = [&](int kb, int buf) {
    unsigned char* kd = smem + buf * (KBLK + VBLK);
#pragma unroll
    for (int s = 0; s < KPW; ++s) {
      const int pc = w * KPW + s, lin = pc * 64 + lane, r = lin / NCK, ch = (lin % NCK) ^ swz<NCK>(r);
      const int key = min(kb * BKV + r, lim - 1);  // clamped rows are masked in the softmax
      const bf16_raw* src = ch < DK / 8 ? kvb + (size_t)key * ldkv + ch * 8 : rotb + (size_t)key * cw + (ch - DK / 8) * 8;
      glds16(src, kd + pc * 1024);
    }
#pragma unroll
    for (int s = 0; s < VPW; ++s) {
      const int pc = w * VPW + s, lin = pc * 64 + lane, r = lin / NCV, ch = (lin % NCV) ^ swz<NCV>(r);
      const int key = min(kb * BKV + r, lim - 1);
      glds16(kvb + (size_t)key * ldkv + DK + ch * 8, kd + KBLK + pc * 1024);
    }
  };

  f32x4_t o[DT];
#pragma unroll
  for (int d = 0; d < DT; ++d) o[d] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  float m_run = -INFINITY, l_run = 0.f;
  int k_off[KF], v_off[DT];
#pragma unroll
  for (int kf = 0; kf < KF; ++kf) k_off[kf] = sw_off<NCK>(l16, kf * 4 + g);
  const int key_lo = 4 * g + (l16 >> 2);
#pragma unroll
  for (int d = 0; d < DT; ++d) v_off[d] = sw_off<NCV>(key_lo, 2 * d + ((l16 & 3) >> 1)) + 8 * (l16 & 1);

  if (nkb > kb_first) stage(kb_first, kb_first & 1);
  for (int kb = kb_first; kb < nkb; ++kb) {
    asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
    if (kb + 1 < nkb) stage(kb + 1, (kb + 1) & 1);
    if (kb * BKV >= wave_lim || (kb + 1) * BKV <= wave_first) continue;
    const unsigned char* ks = smem + (kb & 1) * (KBLK + VBLK);
    const unsigned char* vs = ks + KBLK;
    f32x4_t s[4];
#pragma unroll
    for (int kt = 0; kt < 4; ++kt) {
      s[kt] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kf = 0; kf < KF; ++kf) {
        const u32x4_t k = *reinterpret_cast<const u32x4_t*>(ks + kt * 16 * (KD * 2) + k_off[kf]);
        s[kt] = mfma16(k, qf[kf], s[kt]);
      }
    }
    float mx = -INFINITY;
    if ((kb + 1) * BKV <= wave_min_lim && kb * BKV >= wave_max_first) {
#pragma unroll
      for (int kt = 0; kt < 4; ++kt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          s[kt][r] *= sl2;
          mx = fmaxf(mx, s[kt][r]);
        }
    } else {
#pragma unroll
      for (int kt = 0; kt < 4; ++kt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int key = kb * BKV + kt * 16 + g * 4 + r;
          const float v = key < my_lim && key >= my_first ? s[kt][r] * sl2 : -INFINITY;
          s[kt][r] = v;
          mx = fmaxf(mx, v);
        }
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    const float m_new = fmaxf(m_run, mx);
    const float m_use = m_new == -INFINITY ? 0.f : m_new;
    const float alpha = __builtin_amdgcn_exp2f(m_run - m_use);
    float psum = 0.f;
#pragma unroll
    for (int kt = 0; kt < 4; ++kt)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float p = __builtin_amdgcn_exp2f(s[kt][r] - m_use);
        s[kt][r] = p;
        psum += p;
      }
    l_run = l_run * alpha + psum;
    if (__builtin_amdgcn_ballot_w64(m_new != m_run)) {
#pragma unroll
      for (int d = 0; d < DT; ++d) o[d] *= alpha;
    }
    m_run = m_new;
#pragma unroll
    for (int f2 = 0; f2 < 2; ++f2) {
      float pf[8];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        pf[r] = s[2 * f2][r];
        pf[4 + r] = s[2 * f2 + 1][r];
      }
      const u32x4_t b = pack8(pf);
#pragma unroll
      for (int d = 0; d < DT; ++d) {
        const v4s_t lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
            (__attribute__((address_space(3))) v4s_t*)(vs + f2 * 32 * (DV * 2) + v_off[d]));
        const v4s_t hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
            (__attribute__((address_space(3))) v4s_t*)(vs + (f2 * 32 + 16) * (DV * 2) + v_off[d]));
        u32x4_t c;
        c[0] = __builtin_bit_cast(u32x2_t, lo)[0];
        c[1] = __builtin_bit_cast(u32x2_t, lo)[1];
        c[2] = __builtin_bit_cast(u32x2_t, hi)[0];
        c[3] = __builtin_bit_cast(u32x2_t, hi)[1];
        o[d] = mfma16(c, b, o[d]);
      }
    }
  }

  l_run += __shfl_xor(l_run, 16, 64);
  l_run += __shfl_xor(l_run, 32, 64);
  if (!row_ok) return;
  if (m_run > -INFINITY) l_run += lat_sink(a, head, m_run);
  const float inv = l_run > 0.f ? 1.f / l_run : 0.f;
  const size_t row = tile.row0 + my_row;
  const bf16_raw* gr = gate ? gate + row * ldg + (size_t)head * DV : nullptr;
  bf16_raw* orow = out + row * ldo + (size_t)head * DV;
#pragma unroll
  for (int d = 0; d < DT; ++d) {  // this lane: O[row][d * 16 + 4 g + r]
    f32x4_t v = o[d] * inv;
    if (gr) {
      const u32x2_t gb = *reinterpret_cast<const u32x2_t*>(gr + d * 16 + g * 4);
      v[0] *= sigmoid(__uint_as_float(gb[0] << 16));
      v[1] *= sigmoid(__uint_as_float(gb[0] & 0xffff0000u));
      v[2] *= sigmoid(__uint_as_float(gb[1] << 16));
      v[3] *= sigmoid(__uint_as_float(gb[1] & 0xffff0000u));
    }
    st4(orow + d * 16 + g * 4, v);
  }
}

}  // namespace

// tiles: n_tiles LatTile {row0, nrows <= 128, kv0, pos0, kvlen, base, pad x2} with kv0 + kvlen inside kv and lat
extern "C" int lsa_latent_prefill(const LatentArgs* a, const void* tiles, int n_tiles, const void* q, int ldq,
                                  const void* kv, int ldkv, const void* lat, const void* gate, int ldg, void* out,
                                  int ldo, hipStream_t s) {
  if (!a || n_tiles < 1 || a->window < 0 || a->heads < 1 || a->rp != RP || a->rot_dim < 2 || a->rot_dim > RP || a->rot_dims < 2 ||
      a->rot_dims % 2 || a->rot_dims > a->rot_dim || !a->cos_t || !a->sin_t || a->krp % 64)
    return LSA_BAD_SHAPE;
  if (ldq < a->heads * (a->dkp + RP) || ldq % 8 || ldkv < a->heads * (a->dkp + a->dvp) || ldkv % 8 ||
      ldo < a->heads * a->dvp || ldo % 4 || (gate && (ldg % 4 || (uintptr_t)gate % 8)))
    return LSA_BAD_SHAPE;
  if (((uintptr_t)q | (uintptr_t)kv | (uintptr_t)lat) % 16 || (uintptr_t)out % 8) return LSA_BAD_SHAPE;
  const dim3 grid(n_tiles * a->heads), block(NTHR);
#define LSA_P(K, V)                                                                                                     \
  if (a->dkp == K && a->dvp == V) {                                                                                     \
    latent_prefill_kernel<K, V><<<grid, block, 0, s>>>(*a, (const LatTile*)tiles, (const bf16_raw*)q, ldq,              \
                                                       (const bf16_raw*)kv, ldkv, (const bf16_raw*)lat,                 \
                                                       (const bf16_raw*)gate, ldg, (bf16_raw*)out, ldo);                \
    LSA_CHECK_LAUNCH();                                                                                                 \
    return LSA_OK;                                                                                                      \
  }
  LSA_P(64, 64) LSA_P(64, 128) LSA_P(128, 64) LSA_P(128, 128)
#undef LSA_P
  return LSA_UNSUPPORTED;
}
