// Matrix memory of prompt portions in chunks of 64 rows (mlstm.h), bf16. With F_t the sum of the chunk's log forget
// gates up to row t, g_s = i_s - F_s, (S, n, m) the state before the chunk and M_t = max(m, max_{s <= t} g_s):
//
//   m_t = F_t + M_t
//   S_t^T q = exp(m - M_t) S^T q + sum_{s <= t} exp(g_s - M_t) (k_s . q) v_s       (n_t . q: the same with 1 for v_s)
//   S  <- exp(m - M_e) S + sum_s exp(g_s - M_e) k_s v_s^T                           (e: the chunk's last row)
//
// No exponent is positive. F, g and the maxima of g within a chunk are made by a kernel of their own (one wave per chunk
// and head). Then one workgroup per (segment of a run, head, value slice) walks the segment's chunks with its part of the
// state in accumulators. Where a launch has few workgroups a run is cut into segments: a first launch makes what each
// segment adds to the state, from an empty one (m = -inf); in the second every segment starts from the sum of what lies
// before it. Read-outs go to memory in fp32; a last kernel norms and gates them.
//
// The products run on MFMA: q, k and v are bf16 already, fp32 operands (weights, state, weighted keys) are pairs of bf16.
#include "mfma_pair.h"
#include "mlstm.h"

namespace {

constexpr int C = 64, NT = 512;  // eight waves: four tiles of 16 queries x two halves of the value slice

struct MlItem {  // Mirrored by llm_sharding_amd/ops/retention.py::segments
  int row0, n, slot, pos0;  // the segment's rows
  int ws;                   // the run's first entry in the workspace: its initial state, then its segments' sums
  int seg, n_seg, len;      // which segment; all but the last have len rows
};

// Gates of every row, [g, M, F][heads][rows]: F sums of log forget gates within the chunk, g = i - F, M maxima of g so far
struct MlGates {
  float* all;
  int rows;
};

// Workspace of several segments per run, by entry
struct MlParts {
  float* S;  // [heads][dk][dv]
  float* n;  // [heads][copies][dk]
  float* m;  // [heads][copies][2]: m, and the sum of the segment's log forget gates
};

// grid (items, chunks of an item, groups of 4 heads): one wave per head, one lane per row
__global__ __launch_bounds__(256) void ml_gates_kernel(MlArgs a, const MlItem* __restrict__ items, MlGates G) {
  const MlItem it = items[blockIdx.x];
  const int c0 = blockIdx.y * C, lane = threadIdx.x & 63, h = blockIdx.z * 4 + (threadIdx.x >> 6);
  if (c0 >= it.n || h >= a.heads) return;
  const bool in = c0 + lane < it.n;
  const int row = it.row0 + min(c0 + lane, it.n - 1);
  const float i = ml_input_gate(a, row, h);
  float F = in ? ml_forget_gate(a, row, h) : 0.f;
#pragma unroll
  for (int o = 1; o < 64; o <<= 1) {
    const float x = __shfl_up(F, o, 64);
    F += lane >= o ? x : 0.f;
  }
  const float g = i - F;
  float M = in ? g : -INFINITY;
#pragma unroll
  for (int o = 1; o < 64; o <<= 1) {
    const float x = __shfl_up(M, o, 64);
    M = lane >= o ? fmaxf(M, x) : M;
  }
  if (!in) return;
  const size_t one = (size_t)a.heads * G.rows;
  float* at = G.all + (size_t)h * G.rows + row;
  at[0] = g;
  at[one] = M;
  at[2 * one] = F;
}

template <int DK, int VS>
__global__ __launch_bounds__(NT, 2) void ml_chunk_kernel(MlArgs a, const MlItem* __restrict__ items, MlGates G, MlParts P,
                                                          float* __restrict__ o32, int ldo32, int local) {
  constexpr int KF = DK / 32, VT = VS / 16, TILES = (DK / 16) * VT, MY = (TILES + 7) / 8, VH = VT / 2;
  static_assert(VT % MY == 0, "a wave's tiles are of one row of tiles");
  constexpr int LK = DK + 8, LC = C + 8;  // padded rows: 16-byte reads of 16 rows meet every bank
  constexpr int QB = C * LK, KT = DK * LC, VB = VS * LC, SB = VS * LK;
  __shared__ __attribute__((aligned(16))) bf16_raw smem[2 * QB + 2 * KT + VB + 2 * SB];
  __shared__ __attribute__((aligned(16))) float s_n[DK], s_c[3 * C];  // n; g, M and F of the chunk's rows
  bf16_raw *qh = smem, *kh = qh + QB, *th = kh + QB, *tl = th + KT, *vt_ = tl + KT, *sh = vt_ + VB, *sl = sh + SB;
  const MlItem it = items[blockIdx.x];
  if (local && it.seg == it.n_seg - 1) return;
  const int slices = a.dv / VS, h = blockIdx.y / slices, slice = blockIdx.y % slices, v0 = slice * VS;
  const int tid = threadIdx.x, lane = tid & 63, l16 = lane & 15, q4 = lane >> 4;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int w4 = w & 3, wh = w >> 2;  // tile of queries; half of the value slice, and what the wave stages: q and v, k
  const bf16_raw* in = (const bf16_raw*)a.in + (size_t)it.row0 * a.ldi;
  const size_t one = (size_t)a.heads * G.rows;
  const float *gg = G.all + (size_t)h * G.rows + it.row0, *gM = gg + one, *gF = gM + one;
  const size_t entry = (size_t)a.heads * DK * a.dv, part = (size_t)h * DK * a.dv + v0;
  const size_t nentry = (size_t)a.heads * a.copies, npart = (size_t)h * a.copies + slice;
  const int dv = a.dv;

  // this wave's state tiles: t = w MY + i -> rows (t / VT) 16, channels (t % VT) 16; and these rows of n (in every column)
  const int rt = w * MY / VT;
  const bool mine = w * MY < TILES, owner = mine && (w * MY) % VT == 0;
  f32x4_t S[MY], N = {0.f, 0.f, 0.f, 0.f};
  float m0 = local ? -INFINITY : 0.f, fsum = 0.f;
#pragma unroll
  for (int i = 0; i < MY; ++i) S[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  auto each = [&](auto f) {  // f(accumulator, offset of its first value in a head's [DK][dv])
#pragma unroll
    for (int i = 0; i < MY; ++i) {
      const int t = w * MY + i;
      if (t < TILES) f(S[i], (size_t)((t / VT) * 16 + q4 * 4) * a.dv + (t % VT) * 16 + l16);
    }
  };
  const bool fresh = it.pos0 == it.seg * it.len;  // the run starts at position 0
  float *st = a.S + (size_t)it.slot * entry + part, *stn = a.n + ((size_t)it.slot * nentry + npart) * DK + rt * 16 + q4 * 4,
        *stm = a.m + (size_t)it.slot * nentry + npart;
  // this workgroup's part of the workspace; entry e of the run lies e entries behind
  float *ws = P.S + (size_t)it.ws * entry + part, *wn = P.n + ((size_t)it.ws * nentry + npart) * DK + rt * 16 + q4 * 4,
        *wm = P.m + ((size_t)it.ws * nentry + npart) * 2;
  if (local) {
    if (it.seg == 0) {  // the state before the run, for the second launch
      each([&](f32x4_t&, size_t o) {
#pragma unroll
        for (int r = 0; r < 4; ++r) ws[o + (size_t)r * dv] = fresh ? 0.f : st[o + (size_t)r * dv];
      });
      if (owner && l16 == 0) {
#pragma unroll
        for (int r = 0; r < 4; ++r) wn[r] = fresh ? 0.f : stn[r];
      }
      if (tid == 0) wm[0] = fresh ? 0.f : *stm;
    }
  } else if (it.n_seg == 1) {
    if (!fresh) {
      each([&](f32x4_t& s, size_t o) {
#pragma unroll
        for (int r = 0; r < 4; ++r) s[r] = st[o + (size_t)r * dv];
      });
      if (mine) N = *reinterpret_cast<const f32x4_t*>(stn);
      m0 = *stm;
    }
  } else {
    for (int e = 0; e <= it.seg; ++e) {  // entry 0: before the run, e: what segment e - 1 added
      const float me = wm[e * nentry * 2], fm = e ? m0 + wm[e * nentry * 2 + 1] : -INFINITY, mn = fmaxf(fm, me);
      const float keep = e ? __expf(fm - mn) : 0.f, add = __expf(me - mn);
      const float* src = ws + e * entry;
      each([&](f32x4_t& s, size_t o) {
#pragma unroll
        for (int r = 0; r < 4; ++r) s[r] = fmaf(src[o + (size_t)r * dv], add, s[r] * keep);
      });
      if (mine) N = N * keep + *reinterpret_cast<const f32x4_t*>(wn + e * nentry * DK) * add;
      m0 = mn;
    }
  }

  // Staging: a thread has 16 values of q or k of two neighbouring rows; beside q, 8 values of v of two neighbouring rows
  constexpr int NU = DK / 16, UL = NU < 4 ? NU : 4, RL = 64 / UL, UG = NU / UL;
  const int u = (w4 % UG) * UL + lane % UL, rp = (w4 / UG) * RL + lane / UL;
  const bool on = rp < C / 2 && (wh == 1 || !local);
  constexpr int VU = VS / 8, VG = VU / 4;  // VS 32: 1, 64: 2
  const int vu = (w4 % VG) * 4 + (lane & 3), vr = (w4 / VG) * 16 + (lane >> 2);
  const bool von = vr < C / 2 && wh == 0;
  const bf16_raw* src = in + (wh ? a.ok : a.oq) + h * DK + u * 16;
  u32x4_t rx[2][2], rv[2];
  float rg[2], r1 = 0.f, fend = 0.f, mend = 0.f;
  auto fetch = [&](int c0) {
    const u32x4_t z = {0u, 0u, 0u, 0u};
#pragma unroll
    for (int x = 0; x < 2; ++x) {
      const int r = c0 + 2 * rp + x;
      rx[x][0] = rx[x][1] = z;
      rg[x] = -INFINITY;  // rows past the end weigh nothing
      if (on && r < it.n) {
        const bf16_raw* p = src + (size_t)r * a.ldi;
        rx[x][0] = ld16(p);
        rx[x][1] = ld16(p + 8);
        if (wh) rg[x] = gg[r];
      }
      const int q = c0 + 2 * vr + x;
      rv[x] = z;
      if (von && q < it.n) rv[x] = ld16(in + (size_t)q * a.ldi + a.ov + h * dv + v0 + vu * 8);
    }
    const int e = min(c0 + C, it.n) - 1;
    fend = gF[e];
    mend = gM[e];
    if (tid < 3 * C) {  // waves 0, 1, 2: g, M, F of the chunk's rows
      r1 = c0 + lane < it.n ? gg[w * one + c0 + lane] : w == 0 ? -INFINITY : 0.f;
    }
  };
  auto put = [&](float Me) {  // what was fetched -> LDS; Me: M of the chunk's last row
    if (on) {
      bf16_raw* dh = wh ? kh : qh;
      if (!local) {
#pragma unroll
        for (int x = 0; x < 2; ++x)
#pragma unroll
          for (int y = 0; y < 2; ++y) st16(dh + (2 * rp + x) * LK + u * 16 + 8 * y, rx[x][y]);
      }
      if (wh) {  // k_s exp(g_s - M_e), token by token in accumulator order
        const int vi = vidx(2 * rp);
        const float f0 = __expf(rg[0] - Me), f1 = __expf(rg[1] - Me);
#pragma unroll
        for (int y = 0; y < 2; ++y) {
          float k0[8], k1[8];
          unpack8(rx[0][y], k0);
          unpack8(rx[1][y], k1);
#pragma unroll
          for (int j = 0; j < 8; ++j) {
            unsigned hh, ll;
            split2(k0[j] * f0, k1[j] * f1, hh, ll);
            const int at = (u * 16 + 8 * y + j) * LC + vi;
            *reinterpret_cast<unsigned*>(th + at) = hh;
            *reinterpret_cast<unsigned*>(tl + at) = ll;
          }
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
    if (!local) {
      if (tid < 3 * C) s_c[tid] = r1;
      if (owner && l16 == 0) *reinterpret_cast<f32x4_t*>(s_n + rt * 16 + q4 * 4) = N;
    }
  };

  const int qi = w4 * 16 + l16;
  const u32x4_t ones = {0x3f803f80u, 0x3f803f80u, 0x3f803f80u, 0x3f803f80u};
  fetch(0);
  for (int c0 = 0; c0 < it.n; c0 += C) {
    const int n = min(C, it.n - c0);
    const float Me = fmaxf(m0, mend), dn = __expf(m0 - Me), mb = m0;  // mb: m before the chunk
    m0 = fend + Me;
    fsum += fend;
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();  // the chunk before has been read
    asm volatile("" ::: "memory");
    put(Me);
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
      u32x4_t fh[KF];
      float nq = 0.f;
#pragma unroll
      for (int kf = 0; kf < KF; ++kf) {
        fh[kf] = ld16(qh + qi * LK + kf * 32 + q4 * 8);
        const f32x4_t n0 = *reinterpret_cast<const f32x4_t*>(s_n + kf * 32 + q4 * 8),
                      n1 = *reinterpret_cast<const f32x4_t*>(s_n + kf * 32 + q4 * 8 + 4);
        float q[8];
        unpack8(fh[kf], q);
#pragma unroll
        for (int j = 0; j < 4; ++j) nq = fmaf(q[4 + j], n1[j], fmaf(q[j], n0[j], nq));
      }
      const float Mq = fmaxf(mb, s_c[C + qi]), dq = a.q_scale * __expf(mb - Mq);
      nq *= dq;
      f32x4_t o[VH];
#pragma unroll
      for (int t = 0; t < VH; ++t) {
        o[t] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kf = 0; kf < KF; ++kf) {
          const int at = ((wh * VH + t) * 16 + l16) * LK + kf * 32 + q4 * 8;
          o[t] = mfma16(ld16(sh + at), fh[kf], o[t]);
          o[t] = mfma16(ld16(sl + at), fh[kf], o[t]);
        }
        o[t] *= dq;
      }
      f32x4_t s[4];
#pragma unroll
      for (int kt = 0; kt < 4; ++kt) {
        s[kt] = f32x4_t{0.f, 0.f, 0.f, 0.f};
        if (kt > w4) continue;
#pragma unroll
        for (int kf = 0; kf < KF; ++kf) s[kt] = mfma16(ld16(kh + (kt * 16 + l16) * LK + kf * 32 + q4 * 8), fh[kf], s[kt]);
        const f32x4_t g = *reinterpret_cast<const f32x4_t*>(s_c + kt * 16 + q4 * 4);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          // (what the row does not see: exp(-inf))
          const float p = s[kt][r] * a.q_scale * __expf(kt * 16 + q4 * 4 + r <= qi ? g[r] - Mq : -INFINITY);
          s[kt][r] = p;
          nq += p;
        }
      }
      nq += lane_xor<16>(nq);
      nq += lane_xor<32>(nq);
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
        const float inv = 1.f / ml_denominator(nq, s_c[2 * C + qi] + Mq);
        float* dst = o32 + (size_t)(it.row0 + c0 + qi) * ldo32 + h * dv + v0 + wh * VH * 16 + q4 * 4;
#pragma unroll
        for (int t = 0; t < VH; ++t) *reinterpret_cast<f32x4_t*>(dst + t * 16) = o[t] * inv;
      }
    }
    if (mine) {
      u32x4_t kw[2][2];
#pragma unroll
      for (int f = 0; f < 2; ++f) {
        const int at = (rt * 16 + l16) * LC + f * 32 + q4 * 8;
        kw[f][0] = ld16(th + at);
        kw[f][1] = ld16(tl + at);
      }
      N *= dn;
#pragma unroll
      for (int f = 0; f < 2; ++f) {
        N = mfma16(kw[f][0], ones, N);
        N = mfma16(kw[f][1], ones, N);
      }
#pragma unroll
      for (int i = 0; i < MY; ++i) {
        S[i] *= dn;
#pragma unroll
        for (int f = 0; f < 2; ++f) {
          const u32x4_t x = ld16(vt_ + (((w * MY + i) % VT) * 16 + l16) * LC + f * 32 + q4 * 8);
          S[i] = mfma16(kw[f][0], x, S[i]);
          S[i] = mfma16(kw[f][1], x, S[i]);
        }
      }
    }
  }
  if (local || it.seg == it.n_seg - 1) {
    const size_t e = 1 + it.seg;
    if (local) {
      st = ws + e * entry;
      stn = wn + e * nentry * DK;
      stm = wm + e * nentry * 2;
    }
    each([&](f32x4_t& s, size_t o) {
#pragma unroll
      for (int r = 0; r < 4; ++r) st[o + (size_t)r * dv] = s[r];
    });
    if (owner && l16 == 0) *reinterpret_cast<f32x4_t*>(stn) = N;
    if (tid == 0) {
      stm[0] = m0;
      if (local) stm[1] = fsum;
    }
  }
}

// read-outs -> normed, weighted, gated output: one workgroup per row, dv / 8 lanes per head
__global__ __launch_bounds__(256) void ml_gate_kernel(MlArgs a, const MlItem* __restrict__ items, const float* __restrict__ o32,
                                                      int ldo32) {
  const MlItem it = items[blockIdx.x];
  if ((int)blockIdx.y >= it.n) return;
  const size_t row = it.row0 + blockIdx.y;
  const int g8 = a.dv / 8, n = a.heads * g8;
  for (int c0 = 0; c0 < n; c0 += 256) {
    const int c = c0 + threadIdx.x;
    if (c - (c % g8) >= n) return;  // whole heads leave together
    const float *src = o32 + row * ldo32 + c * 8, *nw = a.norm + c * 8;
    const f32x4_t x0 = *reinterpret_cast<const f32x4_t*>(src), x1 = *reinterpret_cast<const f32x4_t*>(src + 4);
    const f32x4_t n0 = *reinterpret_cast<const f32x4_t*>(nw), n1 = *reinterpret_cast<const f32x4_t*>(nw + 4);
    float x[8] = {x0[0], x0[1], x0[2], x0[3], x1[0], x1[1], x1[2], x1[3]}, g[8], ss = 0.f;
    unpack8(ld16((const bf16_raw*)a.in + row * a.ldi + a.og + c * 8), g);
#pragma unroll
    for (int j = 0; j < 8; ++j) ss = fmaf(x[j], x[j], ss);
    for (int o = g8 / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
    const float rs = 1.f / sqrtf(ss / (float)a.vdim + a.eps);
#pragma unroll
    for (int j = 0; j < 8; ++j) x[j] *= rs * (j < 4 ? n0[j & 3] : n1[j & 3]) * sigmoid(g[j]);
    st16((bf16_raw*)a.out + row * a.ldo + c * 8, pack8(x));
  }
}

}  // namespace

// bf16. items: n_items MlItem (device) of max_rows rows at most; gates: fp32 [3][heads][rows]; several: some run has more
// than one segment, then S / n / m: fp32 entries of heads x (dk x dv / copies x dk / copies x 2); o32 fp32 [rows][ldo32]
extern "C" int lsa_ml_chunked(const MlArgs* a, const void* items, int n_items, int max_rows, int several, float* gates, int rows,
                              float* S, float* n, float* m, float* o32, int ldo32, hipStream_t s) {
  if (bad_ml(a) || !items || n_items < 1 || max_rows < 1 || max_rows > 65535 || rows < 1 || !gates || !o32 ||
      ldo32 < a->heads * a->dv || ldo32 % 4 || (several && (!S || !n || !m)) || a->ldi % 8 || a->ldo % 8 ||
      (a->oq | a->ok | a->ov | a->og) % 8 ||
      ((uintptr_t)a->in | (uintptr_t)a->out | (uintptr_t)a->norm | (uintptr_t)a->n | (uintptr_t)n | (uintptr_t)o32) % 16)
    return LSA_BAD_SHAPE;
  const MlItem* it = (const MlItem*)items;
  const MlGates G{gates, rows};
  const MlParts P{S, n, m};
#define LSA_C(K, V)                                                                                                  \
  if (a->dk == K && (a->dv == V || (V == 64 && a->dv == 128)) && a->copies == a->dv / V) {                           \
    const dim3 grid(n_items, a->heads * (a->dv / V));                                                                \
    ml_gates_kernel<<<dim3(n_items, (max_rows + C - 1) / C, (a->heads + 3) / 4), 256, 0, s>>>(*a, it, G);            \
    if (several) ml_chunk_kernel<K, V><<<grid, NT, 0, s>>>(*a, it, G, P, o32, ldo32, 1);                             \
    ml_chunk_kernel<K, V><<<grid, NT, 0, s>>>(*a, it, G, P, o32, ldo32, 0);                                          \
    ml_gate_kernel<<<dim3(n_items, max_rows), 256, 0, s>>>(*a, it, o32, ldo32);                                      \
    LSA_CHECK_LAUNCH();                                                                                              \
    return LSA_OK;                                                                                                   \
  }
  LSA_C(32, 32) LSA_C(32, 64) LSA_C(64, 32) LSA_C(64, 64) LSA_C(128, 32) LSA_C(128, 64)
#undef LSA_C
  return LSA_UNSUPPORTED;
}
