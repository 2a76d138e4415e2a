// Retention of prompt portions in chunks of 64 rows (retention.h), bf16. With l the decay, rows i, j of a chunk and S
// the state before it:
//
//   o_i = l^(i+1) S^T q_i + sum_{j <= i} l^(i-j) (k_j . q_i) v_j
//   S  <- l^n S + sum_j l^(n-1-j) k_j v_j^T                          (n rows)
//
// One workgroup per (segment of a run, head, value slice) walks the segment's chunks with its part of the state in
// accumulators. Where a launch has few workgroups a run is cut into segments: a first launch makes what each segment
// adds to the state, from zero; in the second every segment starts from the sum of what lies before it.
// The read-outs go to memory in fp32; a last kernel norms and gates them.
//
// The products run on MFMA with every fp32 operand (rotated q and k, weights, state) as a pair of bf16, its rounding
// and the rounding of what that leaves; v is bf16 already. No exponent of a decay is negative.
#include "mfma_pair.h"
#include "retention.h"

namespace {

constexpr int C = 64;

struct RetItem {  // Mirrored by llm_sharding_amd/ops/retention.py::segments
  int row0, n, slot, pos0;  // the segment's rows
  int ws;                   // the run's first entry in the workspace: its initial state, then its segments' sums
  int seg, n_seg, len;      // which segment; all but the last have len rows
};

constexpr int NT = 512;  // eight waves: four tiles of 16 queries x two halves of the value slice

template <int DK, int VS>
__global__ __launch_bounds__(NT, 2) void ret_chunk_kernel(RetArgs a, const RetItem* __restrict__ items, float* ws,
                                                           float* __restrict__ o32, int ldo32, int local) {
  constexpr int KF = DK / 32, VT = VS / 16, TILES = (DK / 16) * VT, MY = (TILES + 7) / 8, VH = VT / 2;
  constexpr int LK = DK + 8, LC = C + 8;  // padded rows: 16-byte reads of 16 rows meet every bank
  constexpr int QB = C * LK, KT = DK * LC, VB = VS * LC, SB = VS * LK;
  __shared__ __attribute__((aligned(16))) bf16_raw smem[4 * QB + 2 * KT + VB + 2 * SB];
  bf16_raw *qh = smem, *ql = qh + QB, *kh = ql + QB, *kl = kh + QB, *th = kl + QB, *tl = th + KT, *vt_ = tl + KT,
           *sh = vt_ + VB, *sl = sh + SB;
  const RetItem it = items[blockIdx.x];
  if (local && it.seg == it.n_seg - 1) return;
  const int slices = a.dv / VS, h = blockIdx.y / slices, v0 = (blockIdx.y % slices) * VS;
  const int tid = threadIdx.x, lane = tid & 63, l16 = lane & 15, q4 = lane >> 4;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int w4 = w & 3, wh = w >> 2;  // tile of queries; half of the value slice, and what the wave stages: q and v, k
  const float l2 = log2f(a.decay[h]);
  const bf16_raw* in = (const bf16_raw*)a.in + (size_t)it.row0 * a.ldi;
  const size_t entry = (size_t)a.heads * DK * a.dv, part = (size_t)h * DK * a.dv + v0;

  // this wave's state tiles: t = w MY + i -> rows (t / VT) 16, channels (t % VT) 16
  f32x4_t S[MY];
#pragma unroll
  for (int i = 0; i < MY; ++i) S[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  auto each = [&](auto f) {  // f(accumulator, offset of its first value in a head's [DK][dv])
#pragma unroll
    for (int i = 0; i < MY; ++i) {
      const int t = w * MY + i;
      if (t < TILES) f(S[i], (size_t)((t / VT) * 16 + q4 * 4) * a.dv + (t % VT) * 16 + l16);
    }
  };
  const int dv = a.dv;
  const bool fresh = it.pos0 == it.seg * it.len;  // the run starts at position 0
  float* st = a.state + (size_t)it.slot * entry + part;
  if (local) {
    if (it.seg == 0)  // the state before the run, for the second launch
      each([&](f32x4_t&, size_t o) {
#pragma unroll
        for (int r = 0; r < 4; ++r) ws[(size_t)it.ws * entry + part + o + (size_t)r * dv] = fresh ? 0.f : st[o + (size_t)r * dv];
      });
  } else if (it.n_seg == 1) {
    if (!fresh)
      each([&](f32x4_t& s, size_t o) {
#pragma unroll
        for (int r = 0; r < 4; ++r) s[r] = st[o + (size_t)r * dv];
      });
  } else {
    for (int e = 0; e <= it.seg; ++e) {  // entry 0: before the run, e: what segment e - 1 added
      const float f = exp2f((float)((it.seg - e) * it.len) * l2);
      const float* src = ws + (size_t)(it.ws + e) * entry + part;
      each([&](f32x4_t& s, size_t o) {
#pragma unroll
        for (int r = 0; r < 4; ++r) s[r] = fmaf(src[o + (size_t)r * dv], f, s[r]);
      });
    }
  }

  // Staging: a thread has 16 values of q or k of two neighbouring rows (the two halves of 8 rotated pairs, or 16
  // values behind them); beside q, 8 values of v of two neighbouring rows.
  constexpr int NU = DK / 16, UL = NU < 4 ? NU : 4, RL = 64 / UL, UG = NU / UL;
  const int u = (w4 % UG) * UL + lane % UL, rp = (w4 / UG) * RL + lane / UL;
  const bool on = rp < C / 2 && (wh == 1 || !local);
  const int half = a.rot_dims / 2;
  const bool turn = a.cos && u * 8 < half;
  const int e0 = !a.cos ? u * 16 : turn ? u * 8 : a.rot_dims + (u - half / 8) * 16;
  const int e1 = turn ? half + u * 8 : e0 + 8;
  constexpr int VU = VS / 8, VG = VU / 4;  // VS 32: 1, 64: 2
  const int vu = (w4 % VG) * 4 + (lane & 3), vr = (w4 / VG) * 16 + (lane >> 2);
  const bool von = vr < C / 2 && wh == 0;
  const bf16_raw* src = in + (wh ? a.ok : a.oq) + h * DK;
  u32x4_t rx[2][2], rv[2];
  f32x4_t rc[2][2], rs[2][2];
  auto fetch = [&](int c0) {
    const u32x4_t z = {0u, 0u, 0u, 0u};
#pragma unroll
    for (int x = 0; x < 2; ++x) {
      const int r = c0 + 2 * rp + x;
      rx[x][0] = rx[x][1] = z;
      rc[x][0] = rc[x][1] = rs[x][0] = rs[x][1] = f32x4_t{0.f, 0.f, 0.f, 0.f};  // rows past the end stay 0
      if (on && r < it.n) {
        const bf16_raw* p = src + (size_t)r * a.ldi;
        rx[x][0] = ld16(p + e0);
        rx[x][1] = ld16(p + e1);
        if (turn) {
          const size_t at = (size_t)(it.pos0 + r) * half + u * 8;
#pragma unroll
          for (int y = 0; y < 2; ++y) {
            rc[x][y] = *reinterpret_cast<const f32x4_t*>(a.cos + at + 4 * y);
            rs[x][y] = *reinterpret_cast<const f32x4_t*>(a.sin + at + 4 * y);
          }
        }
      }
      const int q = c0 + 2 * vr + x;
      rv[x] = z;
      if (von && q < it.n) rv[x] = ld16(in + (size_t)q * a.ldi + a.ov + h * dv + v0 + vu * 8);
    }
  };
  // l^(n-1-j) of the two rows staged, n rows in the chunk; of a whole chunk for now
  auto left = [&](int n, int x) { return exp2f((float)max(n - 1 - 2 * rp - x, 0) * l2); };
  float f0 = left(C, 0), f1 = left(C, 1), dn = exp2f((float)C * l2);
  auto put = [&]() {  // what was fetched -> LDS
    if (on) {
      float kk[2][2][8];
      bf16_raw *dh = wh ? kh : qh, *dl = wh ? kl : ql;
      const float f = wh ? a.k_scale : 1.f;
#pragma unroll
      for (int x = 0; x < 2; ++x) {
        float *lo = kk[x][0], *hi = kk[x][1];
        unpack8(rx[x][0], lo);
        unpack8(rx[x][1], hi);
        if (turn) {
#pragma unroll
          for (int j = 0; j < 8; ++j) {
            const float c = rc[x][j / 4][j % 4], s = rs[x][j / 4][j % 4], m = lo[j], n = hi[j];
            lo[j] = m * c - n * s;
            hi[j] = n * c + m * s;
          }
        }
#pragma unroll
        for (int y = 0; y < 2; ++y) {
#pragma unroll
          for (int j = 0; j < 8; ++j) kk[x][y][j] *= f;
          if (!local) {
            u32x4_t sh_, sl_;
            split8(kk[x][y], sh_, sl_);
            const int at = (2 * rp + x) * LK + (y ? e1 : e0);
            st16(dh + at, sh_);
            st16(dl + at, sl_);
          }
        }
      }
      if (wh) {  // k_j l^(n-1-j), token by token in accumulator order
        const int vi = vidx(2 * rp);
#pragma unroll
        for (int y = 0; y < 2; ++y)
#pragma unroll
          for (int j = 0; j < 8; ++j) {
            unsigned hh, ll;
            split2(kk[0][y][j] * f0, kk[1][y][j] * f1, hh, ll);
            const int at = ((y ? e1 : e0) + j) * LC + vi;
            *reinterpret_cast<unsigned*>(th + at) = hh;
            *reinterpret_cast<unsigned*>(tl + at) = ll;
          }
      }
    }
    if (von) {
      const int vi = vidx(2 * vr);
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const unsigned x = rv[0][j / 2] >> (16 * (j & 1)) & 0xffffu, y = rv[1][j / 2] >> (16 * (j & 1)) & 0xffffu;
        *reinterpret_cast<unsigned*>(vt_ + (vu * 8 + j) * LC + vi) = x | (y << 16);
      }
    }
  };

  const int qi = w4 * 16 + l16;
  const float dq = exp2f((float)(qi + 1) * l2);  // l^(i+1) of this lane's query
  float ds[4][4];                                // l^(i-j), 0 for what it does not see
#pragma unroll
  for (int kt = 0; kt < 4; ++kt)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int back = qi - (kt * 16 + q4 * 4 + r);
      ds[kt][r] = back >= 0 ? exp2f((float)back * l2) : 0.f;
    }
  fetch(0);
  for (int c0 = 0; c0 < it.n; c0 += C) {
    const int n = min(C, it.n - c0);
    if (n < C) {
      f0 = left(n, 0);
      f1 = left(n, 1);
      dn = exp2f((float)n * l2);
    }
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();  // the chunk before has been read
    asm volatile("" ::: "memory");
    put();
    if (!local)  // the state, channel by channel
#pragma unroll
      for (int i = 0; i < MY; ++i) {
        const int t = w * MY + i;
        if (t >= TILES) continue;
        unsigned hh[2], ll[2];
        split2(S[i][0], S[i][1], hh[0], ll[0]);
        split2(S[i][2], S[i][3], hh[1], ll[1]);
        const int at = ((t % VT) * 16 + l16) * LK + (t / VT) * 16 + q4 * 4;
        *reinterpret_cast<u32x2_t*>(sh + at) = u32x2_t{hh[0], hh[1]};
        *reinterpret_cast<u32x2_t*>(sl + at) = u32x2_t{ll[0], ll[1]};
      }
    // (a barrier that does not wait for memory: __syncthreads would drain the read-outs' stores)
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
    if (c0 + C < it.n) fetch(c0 + C);  // arrives under this chunk's products
    if (!local && w4 * 16 < n) {
      u32x4_t fh[KF], fl[KF];
#pragma unroll
      for (int kf = 0; kf < KF; ++kf) {
        fh[kf] = ld16(qh + qi * LK + kf * 32 + q4 * 8);
        fl[kf] = ld16(ql + qi * LK + kf * 32 + q4 * 8);
      }
      f32x4_t o[VH];
#pragma unroll
      for (int t = 0; t < VH; ++t) {
        o[t] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kf = 0; kf < KF; ++kf) {
          const int at = ((wh * VH + t) * 16 + l16) * LK + kf * 32 + q4 * 8;
          const u32x4_t xh = ld16(sh + at), xl = ld16(sl + at);
          o[t] = mfma16(xh, fh[kf], o[t]);
          o[t] = mfma16(xh, fl[kf], o[t]);
          o[t] = mfma16(xl, fh[kf], o[t]);
        }
        o[t] *= dq;
      }
      f32x4_t s[4];
#pragma unroll
      for (int kt = 0; kt < 4; ++kt) {
        s[kt] = f32x4_t{0.f, 0.f, 0.f, 0.f};
        if (kt > w4) continue;
#pragma unroll
        for (int kf = 0; kf < KF; ++kf) {
          const int at = (kt * 16 + l16) * LK + kf * 32 + q4 * 8;
          const u32x4_t xh = ld16(kh + at), xl = ld16(kl + at);
          s[kt] = mfma16(xh, fh[kf], s[kt]);
          s[kt] = mfma16(xh, fl[kf], s[kt]);
          s[kt] = mfma16(xl, fh[kf], s[kt]);
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) s[kt][r] *= ds[kt][r];
      }
#pragma unroll
      for (int f = 0; f < 2; ++f) {
        if (2 * f > w4) continue;
        float p[8];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          p[r] = s[2 * f][r];
          p[4 + r] = s[2 * f + 1][r];
        }
        u32x4_t ph, pl;
        split8(p, ph, pl);
#pragma unroll
        for (int t = 0; t < VH; ++t) {
          const u32x4_t x = ld16(vt_ + ((wh * VH + t) * 16 + l16) * LC + f * 32 + q4 * 8);
          o[t] = mfma16(x, ph, o[t]);
          o[t] = mfma16(x, pl, o[t]);
        }
      }
      if (qi < n) {
        float* dst = o32 + (size_t)(it.row0 + c0 + qi) * ldo32 + h * dv + v0 + wh * VH * 16 + q4 * 4;
#pragma unroll
        for (int t = 0; t < VH; ++t) *reinterpret_cast<f32x4_t*>(dst + t * 16) = o[t];
      }
    }
#pragma unroll
    for (int i = 0; i < MY; ++i) {
      const int t = w * MY + i;
      if (t >= TILES) continue;
      S[i] *= dn;
#pragma unroll
      for (int f = 0; f < 2; ++f) {
        const int at = ((t / VT) * 16 + l16) * LC + f * 32 + q4 * 8;
        const u32x4_t x = ld16(vt_ + ((t % VT) * 16 + l16) * LC + f * 32 + q4 * 8);
        S[i] = mfma16(ld16(th + at), x, S[i]);
        S[i] = mfma16(ld16(tl + at), x, S[i]);
      }
    }
  }
  if (local || it.seg == it.n_seg - 1) {
    float* dst = local ? ws + (size_t)(it.ws + 1 + it.seg) * entry + part : st;
    each([&](f32x4_t& s, size_t o) {
#pragma unroll
      for (int r = 0; r < 4; ++r) dst[o + (size_t)r * dv] = s[r];
    });
  }
}

// read-outs -> normed, gated output: one workgroup per row, dv / 8 lanes per head
__global__ __launch_bounds__(256) void ret_gate_kernel(RetArgs a, const RetItem* __restrict__ items,
                                                       const float* __restrict__ o32, int ldo32) {
  const RetItem it = items[blockIdx.x];
  if ((int)blockIdx.y >= it.n) return;
  const size_t row = it.row0 + blockIdx.y;
  const int g8 = a.dv / 8, n = a.heads * g8;
  for (int c0 = 0; c0 < n; c0 += 256) {
    const int c = c0 + threadIdx.x;
    if (c - (c % g8) >= n) return;  // whole heads leave together
    const float* src = o32 + row * ldo32 + c * 8;
    const f32x4_t x0 = *reinterpret_cast<const f32x4_t*>(src), x1 = *reinterpret_cast<const f32x4_t*>(src + 4);
    float x[8] = {x0[0], x0[1], x0[2], x0[3], x1[0], x1[1], x1[2], x1[3]}, g[8], ss = 0.f;
    unpack8(ld16((const bf16_raw*)a.in + row * a.ldi + a.og + c * 8), g);
#pragma unroll
    for (int j = 0; j < 8; ++j) ss = fmaf(x[j], x[j], ss);
    for (int o = g8 / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
    const float rs = a.oscale / sqrtf(ss / (float)a.vdim + a.eps);
#pragma unroll
    for (int j = 0; j < 8; ++j) x[j] *= rs * (g[j] / (1.f + __expf(-g[j])));
    st16((bf16_raw*)a.out + row * a.ldo + c * 8, pack8(x));
  }
}

}  // namespace

// bf16. items: n_items RetItem (device); ws: fp32 entries of heads x dk x dv (with several segments per run);
// o32 fp32 [rows][ldo32]; max_rows: of an item; several: some run has more than one segment
extern "C" int lsa_ret_chunked(const RetArgs* a, const void* items, int n_items, int max_rows, int several, float* ws,
                               float* o32, int ldo32, hipStream_t s) {
  if (bad_ret(a) || !items || n_items < 1 || max_rows < 1 || max_rows > 65535 || !o32 || ldo32 < a->heads * a->dv ||
      ldo32 % 4 || (several && !ws) || (a->cos && (a->rot_dims / 2) % 8) || a->ldi % 8 || a->ldo % 8 ||
      (a->oq | a->ok | a->ov | a->og) % 8 ||
      ((uintptr_t)a->in | (uintptr_t)a->out | (uintptr_t)a->cos | (uintptr_t)a->sin | (uintptr_t)o32) % 16)
    return LSA_BAD_SHAPE;
  const RetItem* it = (const RetItem*)items;
#define LSA_C(K, V)                                                                                \
  if (a->dk == K && (a->dv == V || (V == 64 && a->dv == 128))) {                                   \
    const dim3 grid(n_items, a->heads * (a->dv / V));                                              \
    if (several) ret_chunk_kernel<K, V><<<grid, NT, 0, s>>>(*a, it, ws, o32, ldo32, 1);           \
    ret_chunk_kernel<K, V><<<grid, NT, 0, s>>>(*a, it, ws, o32, ldo32, 0);                        \
    ret_gate_kernel<<<dim3(n_items, max_rows), 256, 0, s>>>(*a, it, o32, ldo32);                   \
    LSA_CHECK_LAUNCH();                                                                            \
    return LSA_OK;                                                                                 \
  }
  LSA_C(32, 32) LSA_C(32, 64) LSA_C(64, 32) LSA_C(64, 64) LSA_C(128, 32) LSA_C(128, 64)
#undef LSA_C
  return LSA_UNSUPPORTED;
}
