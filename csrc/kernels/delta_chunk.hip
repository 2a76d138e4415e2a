// The gated delta rule over prompt portions in chunks of 32 rows (delta.h), bf16 engine.
//
// With G_i the sum of the log decays of rows 0..i of a chunk (per key channel) and S the state before it,
//
//   u = U - W S             U = T (beta v), W = T (beta k e^G), T = (1 + A)^-1
//   o = (q e^G) S + P u     A_ij = beta_i sum_d k_i k_j e^(G_i - G_j) (j < i),  P_ij the same of q_i, k_j (j <= i)
//   S <- e^G_31 S + (k e^(G_31 - G))^T u
//
// delta_chunk_kernel makes W, U, q e^G, k e^(G_31 - G), P and e^G_31 of every (chunk, head) at once;
// delta_scan_kernel then walks a run's chunks, one workgroup per (run, head). No exponent is ever
// positive: the 16 x 16 blocks on the diagonal of A and P take e^(G_i - G_j) pair by pair, the block
// below them splits it at row 15.
//
// Everything is fp32 or, where it is an operand of a matrix product, a pair of bf16 (the value's
// rounding and the rounding of what that leaves): each product is the sum of three, hi hi + hi lo + lo hi.
// The pairs lie in memory in operand order, the K index in the order in which the accumulators hold it,
// so the state never leaves the scan's registers.
#include "delta.h"

namespace {

constexpr int C = 32;

struct DeltaChunk {  // rows row0 .. row0 + n of one run at positions pos0 ..; before: rows of that run ahead of row0
  int row0, n, slot, pos0, before, pad0, pad1, pad2;
};
struct DeltaSpan {  // chunks [chunk0, chunk0 + chunks) of one run, its rows and first position
  int chunk0, chunks, slot, pos0, row0, n, pad0, pad1;
};

template <int DK>
struct Pieces {  // 1-KiB pieces of a (chunk, head) in the workspace; hi ones first
  static constexpr int KF = DK / 32, W = 0, Q = 4 * KF, K = 8 * KF, P = 12 * KF, E = P + 4, U = E + 1;
};

// 8 values -> operand pieces
LSA_DEVICE void put_pair(unsigned char* hi, unsigned char* lo, int at, const float* f) {
  const u32x4_t h = pack8(f);
  float b[8], r[8];
  unpack8(h, b);
#pragma unroll
  for (int j = 0; j < 8; ++j) r[j] = f[j] - b[j];
  st16(hi + at * 16, h);
  st16(lo + at * 16, pack8(r));
}
LSA_DEVICE void split_pair(const float* f, u32x4_t& h, u32x4_t& l) {
  h = pack8(f);
  float b[8], r[8];
  unpack8(h, b);
#pragma unroll
  for (int j = 0; j < 8; ++j) r[j] = f[j] - b[j];
  l = pack8(r);
}
LSA_DEVICE f32x4_t mfma_pair(u32x4_t ah, u32x4_t al, u32x4_t bh, u32x4_t bl, f32x4_t c) {
  return mfma16(al, bh, mfma16(ah, bl, mfma16(ah, bh, c)));
}

// log(1 + e^x) in fp32 on the hardware's exponential and logarithm
LSA_DEVICE float softplus_fast(float x) {
  const float e = __expf(-fabsf(x));
  return fmaxf(x, 0.f) + (e < 0x1p-9f ? e * (1.f - e * (0.5f - e * 0.33333333f)) : __logf(1.f + e));
}
LSA_DEVICE float silu_fast(float x) {
  return x * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(x * -1.4426950408889634f));
}

// Convolution and silu of one channel over the chunk's rows. load() requests its inputs (up to four taps), so
// that a thread can ask for everything it needs before it waits for any of it; run(f) calls f(row, value),
// zero past the last row.
struct ConvRows {
  bf16_raw raw[C];
  float x1, x2, x3;
  int ch, col;

  // the input j rows before row t
  LSA_DEVICE float past(const DeltaArgs& a, const DeltaChunk& ck, int channels, int t, int j) const {
    if (j - t <= ck.before) return bf2f(((const bf16_raw*)a.in)[(size_t)(ck.row0 + t - j) * a.ldi + col]);
    const int p = ck.pos0 + t - j;
    return p < 0 ? 0.f : a.ring[((size_t)ck.slot * a.taps + p % a.taps) * channels + ch];
  }
  LSA_DEVICE void load(const DeltaArgs& a, const DeltaChunk& ck, int channels, int ch_, int col_) {
    ch = ch_;
    col = col_;
    if (a.taps > 4) return;
    const bf16_raw* in = (const bf16_raw*)a.in + (size_t)ck.row0 * a.ldi + col;
#pragma unroll
    for (int t = 0; t < C; ++t) raw[t] = in[(size_t)min(t, ck.n - 1) * a.ldi];
    x1 = a.taps > 1 ? past(a, ck, channels, 0, 1) : 0.f;
    x2 = a.taps > 2 ? past(a, ck, channels, 0, 2) : 0.f;
    x3 = a.taps > 3 ? past(a, ck, channels, 0, 3) : 0.f;
  }
  template <typename F>
  LSA_DEVICE void run(const DeltaArgs& a, const DeltaChunk& ck, int channels, F f) {
    const float* w = a.conv + (size_t)ch * a.taps + a.taps - 1;
    if (a.taps <= 4) {
      const float w0 = w[0], w1 = a.taps > 1 ? w[-1] : 0.f, w2 = a.taps > 2 ? w[-2] : 0.f, w3 = a.taps > 3 ? w[-3] : 0.f;
#pragma unroll
      for (int t = 0; t < C; ++t) {
        const float x = bf2f(raw[t]);
        const float y = silu_fast(fmaf(x3, w3, fmaf(x2, w2, fmaf(x1, w1, x * w0))));
        f(t, t < ck.n ? y : 0.f);
        x3 = x2;
        x2 = x1;
        x1 = x;
      }
    } else {
#pragma unroll
      for (int t = 0; t < C; ++t) {
        float y = 0.f;
        if (t < ck.n) {
          for (int j = 0; j < a.taps; ++j) y = fmaf(past(a, ck, channels, t, j), w[-j], y);
          y = silu_fast(y);
        }
        f(t, y);
      }
    }
  }
};

template <int DK, int DV>
__global__ __launch_bounds__(256) void delta_chunk_kernel(DeltaArgs a, const DeltaChunk* __restrict__ chunks,
                                                          unsigned char* __restrict__ ws) {
  using PC = Pieces<DK>;
  constexpr int KF = DK / 32, LD = DK + 4, LA = C + 4;
  constexpr size_t STRIDE = (size_t)(PC::U + DV / 8) * 1024;
  __shared__ __attribute__((aligned(16))) float sq[C][LD], sk[C][LD], sg[C][LD], sA[C][LA], sP[C][LA];
  __shared__ float su[2 * C], sb[C];
  const DeltaChunk ck = chunks[blockIdx.x];
  const int h = blockIdx.y, kb = h / (a.heads / a.kv_heads), kc = a.kv_heads * a.dim;
  const int channels = 2 * kc + a.heads * a.vdim;
  const int tid = threadIdx.x, lane = tid & 63, l16 = lane & 15, q4 = lane >> 4;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
  unsigned char* out = ws + ((size_t)blockIdx.x * a.heads + h) * STRIDE;

  static_assert(2 * DK <= 256 && DK + DV <= 256, "one channel per thread");
  const int cd = tid % DK, isk = tid / DK;  // thread < 2 DK: channel cd of q / k, and 16 rows of its decay
  ConvRows qk, vc;
  float zz[16];
  if (tid < 2 * DK) {
    const int d = min(cd, a.dim - 1);
    qk.load(a, ck, channels, isk * kc + kb * a.dim + d, (isk ? a.ok : a.oq) + kb * a.dim + d);
    const float* z = a.z + (size_t)ck.row0 * a.ldz + h * a.dim + d;
#pragma unroll
    for (int t = 0; t < 16; ++t) zz[t] = z[(size_t)min(isk * 16 + t, ck.n - 1) * a.ldz];
  }
  if (tid < DV) {
    const int d = min(tid, a.vdim - 1);
    vc.load(a, ck, channels, 2 * kc + h * a.vdim + d, a.ov + h * a.vdim + d);
  }
  if (tid < 2 * DK) {
    auto& dst = isk ? sk : sq;
    qk.run(a, ck, channels, [&](int t, float y) { dst[t][cd] = cd < a.dim ? y : 0.f; });
    const float A = cd < a.dim ? -a.decay[h] * 1.4426950408889634f : 0.f, bias = cd < a.dim ? a.dt_bias[h * a.dim + cd] : 0.f;
    float g = 0.f;  // sums of log2 decays, 16 rows at a time
#pragma unroll
    for (int t = 0; t < 16; ++t) {
      g = isk * 16 + t < ck.n ? fmaf(A, softplus_fast(zz[t] + bias), g) : g;
      sg[isk * 16 + t][cd] = g;
    }
  }
  if (tid < C) sb[tid] = tid < ck.n ? 1.f / (1.f + __expf(-a.in32[(size_t)(ck.row0 + tid) * a.ld32 + a.ob + h])) : 0.f;
  for (int e = tid; e < C * LA; e += 256) (&sA[0][0])[e] = (&sP[0][0])[e] = 0.f;
  __syncthreads();
  {  // unit vectors: four threads per vector
    const int v = tid >> 2, t = v & (C - 1);
    const float* x = v < C ? sq[t] : sk[t];
    float ss = 0.f;
    for (int d = tid & 3; d < DK; d += 4) ss = fmaf(x[d], x[d], ss);
    ss += __shfl_xor(ss, 1, 64);
    ss += __shfl_xor(ss, 2, 64);
    if ((tid & 3) == 0) su[v] = (v < C ? a.q_scale : 1.f) / sqrtf(ss + a.unit_eps);
  }
  for (int e = tid; e < 16 * DK; e += 256) sg[16 + e / DK][e % DK] += sg[15][e % DK];
  __syncthreads();
  for (int e = tid; e < C * DK; e += 256) {
    const int t = e / DK, d = e % DK;
    sq[t][d] *= su[t];
    sk[t][d] *= su[C + t];
  }
  __syncthreads();

  {  // A and P: the two blocks on the diagonal, one pair of rows per thread
    const int r0 = tid >> 4, r1 = tid & 15;
    const int i = r0 >= r1 ? r0 : 16 + r1, j = r0 >= r1 ? r1 : 16 + r0;
    float x = 0.f, y = 0.f;
#pragma unroll 4
    for (int d = 0; d < DK; d += 4) {
      const f32x4_t gi = *reinterpret_cast<const f32x4_t*>(&sg[i][d]), gj = *reinterpret_cast<const f32x4_t*>(&sg[j][d]);
      const f32x4_t ki = *reinterpret_cast<const f32x4_t*>(&sk[i][d]), kj = *reinterpret_cast<const f32x4_t*>(&sk[j][d]);
      const f32x4_t qi = *reinterpret_cast<const f32x4_t*>(&sq[i][d]);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float z = kj[e] * __builtin_amdgcn_exp2f(gi[e] - gj[e]);
        x = fmaf(ki[e], z, x);
        y = fmaf(qi[e], z, y);
      }
    }
    if (i != j) sA[i][j] = sb[i] * x;
    sP[i][j] = y;
    if (tid < 16) {  // the second block's diagonal
      float p = 0.f;
      for (int d = 0; d < DK; ++d) p = fmaf(sq[16 + tid][d], sk[16 + tid][d], p);
      sP[16 + tid][16 + tid] = p;
    }
  }
  if (w < 2) {  // the block below, through row 15: wave 0 A, wave 1 P
    f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
    const auto& sx = w ? sq : sk;
#pragma unroll
    for (int kf = 0; kf < KF; ++kf) {
      float x[8], y[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const int d = kf * 32 + q4 * 8 + e;
        const float g = sg[15][d];
        x[e] = sx[16 + l16][d] * __builtin_amdgcn_exp2f(sg[16 + l16][d] - g);
        y[e] = sk[l16][d] * __builtin_amdgcn_exp2f(g - sg[l16][d]);
      }
      u32x4_t xh, xl, yh, yl;
      split_pair(x, xh, xl);
      split_pair(y, yh, yl);
      acc = mfma_pair(xh, xl, yh, yl, acc);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = 16 + q4 * 4 + r;
      if (w) sP[i][l16] = acc[r];
      else sA[i][l16] = sb[i] * acc[r];
    }
  }
  // q e^G (rows x key channels) and k e^(G_31 - G) (key channels x rows)
  for (int e = tid; e < 2 * KF * 64; e += 256) {
    const int ln = e & 63, kf = (e >> 6) % KF, t = (e >> 6) / KF * 16 + (ln & 15), d0 = kf * 32 + (ln >> 4) * 4;
    float f[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int d = d0 + (j & 4) * 4 + (j & 3);
      f[j] = sq[t][d] * __builtin_amdgcn_exp2f(sg[t][d]);
    }
    put_pair(out + PC::Q * 1024, out + (PC::Q + 2 * KF) * 1024, e, f);
  }
  for (int e = tid; e < 2 * KF * 64; e += 256) {
    const int ln = e & 63, d = (e >> 6) * 16 + (ln & 15), t0 = (ln >> 4) * 4;
    float f[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int t = t0 + (j & 4) * 4 + (j & 3);
      f[j] = sk[t][d] * __builtin_amdgcn_exp2f(sg[C - 1][d] - sg[t][d]);
    }
    put_pair(out + PC::K * 1024, out + (PC::K + 2 * KF) * 1024, e, f);
  }
  for (int d = tid; d < DK; d += 256) reinterpret_cast<float*>(out + PC::E * 1024)[d] = __builtin_amdgcn_exp2f(sg[C - 1][d]);
  __syncthreads();
  if (tid < 128) {  // P (rows x rows)
    const int t = (tid >> 6) * 16 + l16;
    float f[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) f[j] = sP[t][q4 * 4 + (j & 4) * 4 + (j & 3)];
    put_pair(out + PC::P * 1024, out + (PC::P + 2) * 1024, tid, f);
  }
  // (1 + A) x = b, one column per thread: beta v -> U, beta k e^G -> W
  if (tid < DV + DK) {
    const int c = tid;
    float x[C];
    if (c < DV) {
      vc.run(a, ck, channels, [&](int t, float y) { x[t] = c < a.vdim ? y * sb[t] : 0.f; });
    } else {
#pragma unroll
      for (int t = 0; t < C; ++t) x[t] = sb[t] * sk[t][c - DV] * __builtin_amdgcn_exp2f(sg[t][c - DV]);
    }
#pragma unroll
    for (int i = 1; i < C; ++i) {
      float s = x[i];
#pragma unroll
      for (int j = 0; j < i; j += 4) {
        const f32x4_t r = *reinterpret_cast<const f32x4_t*>(&sA[i][j]);
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (j + e < i) s = fmaf(-r[e], x[j + e], s);
      }
      x[i] = s;
    }
    if (c < DV) {
      f32x4_t* u = reinterpret_cast<f32x4_t*>(out + (PC::U + (c / 16) * 2) * 1024);
#pragma unroll
      for (int e = 0; e < 8; ++e) u[e * 16 + (c & 15)] = f32x4_t{x[4 * e], x[4 * e + 1], x[4 * e + 2], x[4 * e + 3]};
    } else {
#pragma unroll
      for (int t = 0; t < C; ++t) sq[t][c - DV] = x[t];  // q is in memory already
    }
  }
  __syncthreads();
  for (int e = tid; e < 2 * KF * 64; e += 256) {
    const int ln = e & 63, kf = (e >> 6) % KF, t = (e >> 6) / KF * 16 + (ln & 15), d0 = kf * 32 + (ln >> 4) * 4;
    float f[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) f[j] = sq[t][d0 + (j & 4) * 4 + (j & 3)];
    put_pair(out, out + 2 * KF * 1024, e, f);
  }
}

LSA_DEVICE void glds16(const void* src, unsigned char* lds_base) {
  __builtin_amdgcn_global_load_lds(src, (__attribute__((address_space(3))) void*)lds_base, 16, 0, 0);
}

// One workgroup per (run, head, NW 16 value channels): the state in registers (a wave has 16 channels of it), a
// chunk's operands by LDS-DMA into a double buffer. Leaves the read-outs in fp32 for delta_norm_kernel.
template <int DK, int DV, int NW>
__global__ __launch_bounds__(NW * 64) void delta_scan_kernel(DeltaArgs a, const DeltaSpan* __restrict__ spans,
                                                             const unsigned char* __restrict__ ws,
                                                             float* __restrict__ o32) {
  using PC = Pieces<DK>;
  constexpr int KF = DK / 32, MT = DK / 16, NP = PC::U;
  constexpr int NDMA = (NP + NW - 1) / NW, LESS = NP % NW;  // DMA instructions per wave; waves >= LESS > 0: one less
  constexpr size_t STRIDE = (size_t)(PC::U + DV / 8) * 1024;
  __shared__ __attribute__((aligned(16))) unsigned char smem[3 * NP * 1024];
  const DeltaSpan sp = spans[blockIdx.x];
  const int h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, l16 = lane & 15, q4 = lane >> 4;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6), vt = blockIdx.z * NW + w;  // this wave's channels: 16 vt ..
  const unsigned char* src = ws + ((size_t)sp.chunk0 * a.heads + h) * STRIDE;
  const size_t step = (size_t)a.heads * STRIDE;

  f32x4_t S[MT], U0[2], U1[2];
  float* st = a.state + ((size_t)sp.slot * a.heads + h) * DK * DV + vt * 16 + l16;
#pragma unroll
  for (int m = 0; m < MT; ++m)
#pragma unroll
    for (int r = 0; r < 4; ++r) S[m][r] = st[(size_t)(m * 16 + q4 * 4 + r) * DV];
  if (sp.pos0 == 0) {
#pragma unroll
    for (int m = 0; m < MT; ++m) S[m] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  }
  auto stage = [&](int c, int buf) {
    const unsigned char* p = src + c * step + lane * 16;
#pragma unroll
    for (int i = 0; i < NDMA; ++i)
      if (LESS == 0 || i * NW + w < NP) glds16(p + (i * NW + w) * 1024, smem + (buf * NP + i * NW + w) * 1024);
  };
  auto load_u = [&](int c, f32x4_t (&U)[2]) {
    const unsigned char* p = src + c * step + (PC::U + vt * 2) * 1024 + lane * 16;
#pragma unroll
    for (int m = 0; m < 2; ++m) U[m] = *reinterpret_cast<const f32x4_t*>(p + m * 1024);
  };
  const int v = vt * 16 + l16;
  float* op = o32 + (size_t)sp.row0 * a.heads * a.vdim + h * a.vdim + min(v, a.vdim - 1);
  const int ldo = a.heads * a.vdim;

  // Chunk c + 2 is requested while chunk c runs: operands into the buffer chunk c - 1 used, U into the
  // registers chunk c's has left. The counted wait leaves those of chunk c + 1 in flight (the read-outs'
  // stores come after them, so it waits for a few of them at most).
  int buf = 0, buf2 = 2;
  auto chunk = [&](int c, f32x4_t (&U)[2]) {
    if (c + 1 < sp.chunks) {
      if (LESS == 0 || w < LESS) asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)" ::"i"(NDMA + 2) : "memory");
      else asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)" ::"i"(NDMA + 1) : "memory");
    } else {
      asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)" ::: "memory");
    }
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
    const unsigned char* p = smem + buf * NP * 1024 + lane * 16;
    // operands are read a whole group ahead of their products; pin() is where the wait for a group goes
    auto fetch = [&](auto& r, int first) {
#pragma unroll
      for (int i = 0; i < (int)(sizeof(r) / sizeof(r[0])); ++i) r[i] = *reinterpret_cast<const u32x4_t*>(p + (first + i) * 1024);
    };
    auto pin = [](auto& r) {
#pragma unroll
      for (int i = 0; i < (int)(sizeof(r) / sizeof(r[0])); ++i) asm volatile("" : "+v"(r[i]));
    };
    u32x4_t wf[4 * KF], qf[4 * KF], kf_[4 * KF], pf[4];
    f32x4_t ef[MT];
    fetch(wf, PC::W);
    fetch(qf, PC::Q);
    float u[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) u[j] = U[j >> 2][j & 3];
#pragma unroll
    for (int j = 0; j < 8; ++j) asm volatile("" : "+v"(u[j]));
    if (c + 2 < sp.chunks) {
      stage(c + 2, buf2);
      load_u(c + 2, U);
    }
    u32x4_t sh[KF], sl[KF];
#pragma unroll
    for (int kf = 0; kf < KF; ++kf) {
      float f[8];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        f[j] = S[2 * kf][j];
        f[4 + j] = S[2 * kf + 1][j];
      }
      split_pair(f, sh[kf], sl[kf]);
    }
    f32x4_t V[2], O[2];
#pragma unroll
    for (int m = 0; m < 2; ++m) V[m] = O[m] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    pin(wf);
#pragma unroll
    for (int kf = 0; kf < KF; ++kf)
#pragma unroll
      for (int m = 0; m < 2; ++m) V[m] = mfma_pair(wf[m * KF + kf], wf[(2 + m) * KF + kf], sh[kf], sl[kf], V[m]);
    fetch(kf_, PC::K);
    fetch(pf, PC::P);
#pragma unroll
    for (int m = 0; m < MT; ++m)
      ef[m] = *reinterpret_cast<const f32x4_t*>(smem + (buf * NP + PC::E) * 1024 + (m * 16 + q4 * 4) * 4);
    pin(qf);
#pragma unroll
    for (int kf = 0; kf < KF; ++kf)
#pragma unroll
      for (int m = 0; m < 2; ++m) O[m] = mfma_pair(qf[m * KF + kf], qf[(2 + m) * KF + kf], sh[kf], sl[kf], O[m]);
    u32x4_t vh, vl;
#pragma unroll
    for (int j = 0; j < 8; ++j) u[j] -= V[j >> 2][j & 3];
    split_pair(u, vh, vl);
    pin(kf_);
    pin(ef);
#pragma unroll
    for (int m = 0; m < MT; ++m) S[m] = mfma_pair(kf_[m], kf_[MT + m], vh, vl, S[m] * ef[m]);
#pragma unroll
    for (int m = 0; m < 2; ++m) {
      O[m] = mfma_pair(pf[m], pf[2 + m], vh, vl, O[m]);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = c * C + m * 16 + q4 * 4 + r;
        if (t < sp.n && v < a.vdim) op[(size_t)t * ldo] = O[m][r];
      }
    }
    buf = buf == 2 ? 0 : buf + 1;
    buf2 = buf2 == 2 ? 0 : buf2 + 1;
  };
  stage(0, 0);
  load_u(0, U0);
  if (sp.chunks > 1) {
    stage(1, 1);
    load_u(1, U1);
  }
  for (int c = 0; c < sp.chunks; c += 2) {
    chunk(c, U0);
    if (c + 1 < sp.chunks) chunk(c + 1, U1);
  }
#pragma unroll
  for (int m = 0; m < MT; ++m)
#pragma unroll
    for (int r = 0; r < 4; ++r) st[(size_t)(m * 16 + q4 * 4 + r) * DV] = S[m][r];
}

// Read-outs -> RMS norm over the head's value channels, weight, output gate. One workgroup per (chunk, head), 16
// lanes per row.
__global__ __launch_bounds__(256) void delta_norm_kernel(DeltaArgs a, const DeltaChunk* __restrict__ chunks,
                                                         const float* __restrict__ o32) {
  const DeltaChunk ck = chunks[blockIdx.x];
  const int h = blockIdx.y, l16 = threadIdx.x & 15;
  for (int t = threadIdx.x >> 4; t < ck.n; t += 16) {
    const size_t row = ck.row0 + t;
    const float* o = o32 + (row * a.heads + h) * a.vdim;
    const bf16_raw* g = (const bf16_raw*)a.gate + row * a.ldg + h * a.vdim;
    bf16_raw* out = (bf16_raw*)a.out + row * a.ldo + h * a.vdim;
    float x[8], ss = 0.f;  // vdim <= 128
    if (a.vdim == 128 && !((a.ldg | a.ldo) & 7) && !(((uintptr_t)a.gate | (uintptr_t)a.out) & 15)) {
      *reinterpret_cast<f32x4_t*>(x) = *reinterpret_cast<const f32x4_t*>(o + l16 * 8);
      *reinterpret_cast<f32x4_t*>(x + 4) = *reinterpret_cast<const f32x4_t*>(o + l16 * 8 + 4);
      float z[8];
      unpack8(ld16(g + l16 * 8), z);
#pragma unroll
      for (int j = 0; j < 8; ++j) ss = fmaf(x[j], x[j], ss);
      const float rs = 1.f / sqrtf(group_sum<16>(ss) / 128.f + a.eps);
#pragma unroll
      for (int j = 0; j < 8; ++j) x[j] *= rs * a.norm[l16 * 8 + j] * sigmoid(z[j]);
      st16(out + l16 * 8, pack8(x));
      continue;
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int d = j * 16 + l16;
      x[j] = d < a.vdim ? o[d] : 0.f;
      ss = fmaf(x[j], x[j], ss);
    }
    const float rs = 1.f / sqrtf(group_sum<16>(ss) / (float)a.vdim + a.eps);
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int d = j * 16 + l16;
      if (d < a.vdim) out[d] = f2bf(x[j] * rs * a.norm[d] * sigmoid(bf2f(g[d])));
    }
  }
}

}  // namespace

// bytes of one (chunk, head) in the workspace, 0: size not built
extern "C" int lsa_delta_chunk_bytes(int dk, int dv) {
  if ((dk != 32 && dk != 64 && dk != 128) || (dv != 32 && dv != 64 && dv != 128)) return 0;
  return (12 * (dk / 32) + 5 + dv / 8) * 1024;
}

// chunks: n_chunks DeltaChunk; spans: n_spans DeltaSpan over them; ws: n_chunks * heads * lsa_delta_chunk_bytes;
// o32: [rows][heads * vdim]
extern "C" int lsa_delta_chunked(const DeltaArgs* a, const void* chunks, int n_chunks, const void* spans, int n_spans,
                                 void* ws, float* o32, hipStream_t s) {
  if (!a || bad_delta(a) || !a->gate || n_chunks < 1 || n_spans < 1 || !chunks || !spans || !ws || !o32 || (uintptr_t)ws % 16)
    return LSA_BAD_SHAPE;
#define LSA_S(K, V, NW)                                                                                                  \
  delta_scan_kernel<K, V, NW><<<dim3(n_spans, a->heads, V / (NW * 16)), NW * 64, 0, s>>>(*a, (const DeltaSpan*)spans,     \
                                                                                       (const unsigned char*)ws, o32)
#define LSA_C(K, V)                                                                                                       \
  if (a->dk == K && a->dv == V) {                                                                                         \
    delta_chunk_kernel<K, V><<<dim3(n_chunks, a->heads), 256, 0, s>>>(*a, (const DeltaChunk*)chunks, (unsigned char*)ws); \
    LSA_CHECK_LAUNCH();                                                                                                   \
    LSA_S(K, V, (V == 32 ? 2 : 4));                                                                                       \
    LSA_CHECK_LAUNCH();                                                                                                   \
    delta_norm_kernel<<<dim3(n_chunks, a->heads), 256, 0, s>>>(*a, (const DeltaChunk*)chunks, o32);                       \
    LSA_CHECK_LAUNCH();                                                                                                   \
    return LSA_OK;                                                                                                        \
  }
  LSA_C(32, 32) LSA_C(32, 64) LSA_C(32, 128) LSA_C(64, 32) LSA_C(64, 64) LSA_C(64, 128) LSA_C(128, 32) LSA_C(128, 64)
  LSA_C(128, 128)
#undef LSA_C
#undef LSA_S
  return LSA_UNSUPPORTED;
}
