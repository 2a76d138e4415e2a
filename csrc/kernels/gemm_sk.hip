// Projection GEMM for > 128 rows (prompt prefill and big decode batches):
//   C[M, N] = A[M, K] @ W^T, bf16 in, fp32 accumulate, with the fused epilogues of epilogue.h
// (RoPE + KV-cache append | SwiGLU | residual add | store), replacing the reference's
// nn.Linear calls inside HF LlamaDecoderLayer (/root/reference/utils/shard_loader.py:66-74).
//
// Structure (cdna_hip_programming.md §5 "The 256² 8-phase template", T1-T5):
//  * 256 x BN output tile (BN = 256 or 128) per 512-thread workgroup (8 waves, 2 per SIMD),
//    K step 64, one workgroup per CU, all LDS in ONE __shared__ array.
//  * Both operands reach LDS by LDS-DMA (global_load_lds_dwordx4): the packed-16x32 weights
//    (common.h) are already one lane-linear 1 KiB block per (16 cols, 32 k) fragment; the A
//    tile is fetched as whole 128-B rows (full cache lines: 5-12 % faster than gathering
//    fragment-order half lines, scripts/sk_ablate.py) into a row-major image whose 16-B chunks
//    are XOR-swizzled by row (per-lane source address), so every MFMA operand read is a
//    conflict-free ds_read_b128.
//  * Each K-tile runs as 4 phases (one output quadrant of 16 or 8 MFMAs each). The two wave
//    groups (waves 0-3 / 4-7, i.e. the two waves of every SIMD) run one raw s_barrier apart, so
//    one wave of a SIMD issues MFMAs while its partner issues LDS reads and DMA.
//  * The DMA for a buffer region is issued 5-6 phases ahead of its first read and retired by a
//    COUNTED s_waitcnt vmcnt (one K-tile of DMA stays in flight across every barrier).
//  * Work is split "data-parallel + stream-K": full rounds of 256-row x BN tiles go one per
//    workgroup (grouped tile order, XCD-aware block remap), the remaining tiles' K iterations
//    are spread evenly over the grid; a tile split between workgroups is combined by the last
//    arriving one (write-through fp32 slabs + an agent-scope ticket, §6 Guideline 16) which
//    then runs the fused epilogue.
//  * Epilogue: accumulators -> LDS (fp32) -> one thread per 16-column tile row -> the
//    vectorised row16 epilogues of epilogue.h (16-B stores).
#include "gemm_sk_core.h"

namespace {

template <int BM, int BN, int EPI, int NB>
__global__ __launch_bounds__(NTHR) void gemm_sk_kernel(const bf16_raw* __restrict__ A, const bf16_raw* __restrict__ W,
                                                        SkParams prm, EpiArgs ep, float* __restrict__ slab,
                                                        unsigned* __restrict__ counters) {
  using K_ = Kern<BM, BN, EPI, NB>;
  __shared__ __attribute__((aligned(16))) unsigned char smem[Geo<BM, BN, NB>::SMEM];
  K_ k;
  k.smem = smem;
  k.A = A;
  k.W = W;
  k.p = &prm;
  k.tid = threadIdx.x;
  k.lane = threadIdx.x & 63;
  k.w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  k.wr = k.w / K_::WN;
  k.wc = k.w % K_::WN;
  k.group = k.w >> 2;
  const int G = prm.G;
  // XCD-aware remap (bijective): blocks that share an XCD get consecutive work ids
  const int hw = blockIdx.x;
  int g;
  {
    const int q = G / 8, r = G % 8, x = hw % 8;
    g = (x < r ? x * (q + 1) : r * (q + 1) + (x - r) * q) + hw / 8;
  }
  f32x4_t acc[K_::FM][K_::FN];
  auto zero = [&]() {
#pragma unroll
    for (int i = 0; i < K_::FM; ++i)
#pragma unroll
      for (int j = 0; j < K_::FN; ++j) acc[i][j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  };

  // One work loop (a single inlined copy of the segment and epilogue code keeps register
  // allocation within 256 VGPRs): first the data-parallel rounds (whole tiles r*G + g), then
  // this workgroup's stream-K iterations [lo, hi) of the remaining tiles' K loops.
  const long long S = (long long)prm.sk_tiles * prm.NKT;
  const long long lo = prm.sk_tiles ? (long long)g * S / G : 0, hi = prm.sk_tiles ? (long long)(g + 1) * S / G : 0;
  int* flag = reinterpret_cast<int*>(smem + Geo<BM, BN, NB>::SMEM - 16);
  int r = 0;
  long long it = lo;
  bool split_done = false;
  // split mode: U = sk_tiles * split work units spread EVENLY over the XCDs (units u, u+1 of
  // one K range - neighbouring tiles that share A or W panels - on one XCD); blocks beyond U idle
  int su = -1;
  if (prm.split) {
    const int U = prm.sk_tiles * prm.split, q = U / 8, rr = U % 8, x = hw % 8, j = hw / 8;
    if (j < (x < rr ? q + 1 : q)) su = (x < rr ? x * (q + 1) : rr * (q + 1) + (x - rr) * q) + j;
  }
  for (;;) {
    int tile, ts = 0, ka = 0, kb = prm.NKT, sp = 0;
    bool sk = false;
    if (r < prm.dp_rounds) {
      tile = r * G + g;
      ++r;
    } else if (prm.split) {
      if (split_done || su < 0) break;
      ts = su % prm.sk_tiles;
      sp = su / prm.sk_tiles;
      ka = sp * prm.NKT / prm.split;
      kb = (sp + 1) * prm.NKT / prm.split;
      tile = prm.dp_rounds * G + ts;
      split_done = true;
    } else if (it < hi) {
      ts = (int)(it / prm.NKT);
      ka = (int)(it - (long long)ts * prm.NKT);
      const long long tile_end = (long long)(ts + 1) * prm.NKT;
      kb = (int)((hi < tile_end ? hi : tile_end) - (long long)ts * prm.NKT);
      tile = prm.dp_rounds * G + ts;
      sk = true;
    } else {
      break;
    }
    const bool partial = ka != 0 || kb != prm.NKT;
    int mt, nt;
    tile_coords(prm, tile, mt, nt);
    zero();
    k.run_segment(acc, mt * BM, nt, ka, kb);
    LSA_STAMP(k.stamp_base + 2);
    bool do_epi = true;
    if (partial && EPI != EPI_PARTIAL) {
      // contributors of this tile, in K order: split mode - workgroups ts + s * sk_tiles
      // (slot 0); stream-K - the workgroups whose iteration ranges intersect the tile's
      const long long t0 = (long long)ts * prm.NKT, t1 = t0 + prm.NKT;
      const int g_first = prm.split ? 0 : (int)(((t0 + 1) * G - 1) / S);
      const int g_last = prm.split ? prm.split - 1 : (int)((t1 * G - 1) / S);
      k.slab_store(slab, prm.split ? (size_t)su * 2 : (size_t)g * 2 + (it == lo ? 0 : 1), acc);
      asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
      __syncthreads();
      if (k.tid == 0) {
        const unsigned old = __hip_atomic_fetch_add(&counters[ts], 1u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        *flag = old == (unsigned)(g_last - g_first);
      }
      __syncthreads();
      LSA_STAMP(k.stamp_base + 3);
      do_epi = *flag != 0;
      if (do_epi) {
        // fixed summation order (bitwise-reproducible results): with two contributors the
        // sum is commutative; with more, every partial - this one's too - is re-read in order
        const bool all = g_last - g_first > 1;
        if (all) zero();
        for (int ci = g_first; ci <= g_last; ++ci) {
          int c, slot;
          if (prm.split) {
            c = ts + ci * prm.sk_tiles;
            slot = 0;
          } else {
            c = ci;
            slot = (long long)c * S / G >= t0 ? 0 : 1;  // slot 0: c's range starts in this tile
          }
          if (c == (prm.split ? su : g) && !all) continue;
          k.slab_add(slab, (size_t)c * 2 + slot, acc);
        }
        if (k.tid == 0) __hip_atomic_store(&counters[ts], 0u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        __syncthreads();  // every wave's slab ring reads are done before the epilogue reuses LDS
      }
    }
    LSA_STAMP(k.stamp_base + 4);
    if (do_epi) k.epilogue(ep, acc, mt * BM, nt, sp);
    LSA_STAMP(k.stamp_base + 5);
    k.stamp_base = k.stamp_base + 6 < 30 ? k.stamp_base + 6 : 24;
    __syncthreads();
    if (sk) it = (long long)ts * prm.NKT + kb;
  }
}

template <int BM, int BN, int EPI, int NB>
int launch(const bf16_raw* A, const bf16_raw* W, const SkParams& prm, const EpiArgs& ep, float* slab,
           unsigned* cnt, hipStream_t s) {
  gemm_sk_kernel<BM, BN, EPI, NB><<<prm.G, NTHR, 0, s>>>(A, W, prm, ep, slab, cnt);
  LSA_CHECK_LAUNCH();
  return LSA_OK;
}

template <int BM, int EPI>
int dispatch(const bf16_raw* A, const bf16_raw* W, const SkParams& prm, const EpiArgs& ep, float* slab,
             unsigned* cnt, int bn, int nb, hipStream_t s) {
  if (bn == 256) {
    if constexpr (BM == 128) {
      if (nb == 3) return launch<BM, 256, EPI, 3>(A, W, prm, ep, slab, cnt, s);
    }
    return launch<BM, 256, EPI, 2>(A, W, prm, ep, slab, cnt, s);
  }
  if (bn == 192) return launch<BM, 192, EPI, 2>(A, W, prm, ep, slab, cnt, s);
  return nb == 3 ? launch<BM, 128, EPI, 3>(A, W, prm, ep, slab, cnt, s)
                 : launch<BM, 128, EPI, 2>(A, W, prm, ep, slab, cnt, s);
}

}  // namespace

// bm: tile height 256 or 128. bn: tile width 256 / 192 (192: N % 16 == 0, partial last tile) / 128.
// nb: DMA ring buffers, 2 or 3 (3 for bn 128, and bn 256 at bm 128; 0 = the default: 3 where
// allowed). grid: workgroups (<= 1024); dp: 1 = whole tiles in data-parallel rounds first (0 =
// all tiles are remainder).
// epi EPI_PARTIAL: every tile split into exactly `split` K ranges (tiles * split <= grid), fp32
// partial k stored to ((float*)ep->out)[k][M][ldo], no slabs or tickets (lsa_resid_rmsnorm_partials sums them).
// split: 0 = remainder by stream-K, S >= 1 = remainder tiles split into up to S K ranges
// (clamped to NKT and to grid / remainder tiles; stream-K when the remainder exceeds the grid).
// slab: >= 2 * grid * bm * bn floats and counters: >= remainder tiles (zeroed) when any tile is
// split. Returns LSA_BAD_SHAPE on any shape the kernel's indexing cannot take.
extern "C" int lsa_gemm_sk(const void* a, int lda, const void* wp, int M, int N, int K, int epi,
                           const EpiArgs* ep, int bm, int bn, int nb, int grid, int dp, int split, int group_m, float* slab,
                           unsigned* counters, long long slab_floats, int n_counters, hipStream_t stream) {
  if (M < 1 || K < BK || K % BK || lda < K || lda % 8 || !ep) return LSA_BAD_SHAPE;
  if (bn != 256 && bn != 192 && bn != 128) return LSA_UNSUPPORTED;
  if (bm != 256 && bm != 128) return LSA_UNSUPPORTED;
  const int BM = bm;
  if (nb == 0) nb = (bn == 128 || (bm == 128 && bn == 256)) ? 3 : 2;
  if (nb != 2 && !(nb == 3 && (bn == 128 || (bm == 128 && bn == 256)))) return LSA_UNSUPPORTED;
  if (bn == 192 ? (N % 16 || (epi_gated(epi) && N % 32)) : N % bn) return LSA_BAD_SHAPE;
  if (grid < 1 || grid > 1024 || group_m < 1) return LSA_BAD_SHAPE;
  if (epi == EPI_RESID && !ep->resid) return LSA_BAD_SHAPE;
  if (epi == EPI_QKV && (!ep->k_cache || !ep->v_cache || !ep->slot || !ep->pos)) return LSA_BAD_SHAPE;
  if (epi == EPI_ARGMAX ? (!ep->keys || bn == 192) : !(ep->out || (epi == EPI_STORE && ep->out32))) return LSA_BAD_SHAPE;
  if (ep->ss_out && (epi != EPI_RESID || bn == 192 || N % 64 || ep->ss_n != N / 64)) return LSA_BAD_SHAPE;
  if (ep->ss_in && ((epi != EPI_QKV && epi != EPI_SWIGLU) || ep->ss_n < 4 || ep->ss_n % 4 || K != 64 * ep->ss_n))
    return LSA_BAD_SHAPE;
  if (epi == EPI_STORE && bad_store(*ep, N)) return LSA_BAD_SHAPE;
  if (epi == EPI_PARTIAL && (split < 1 || ep->ldo < N || ep->ldo % 4)) return LSA_BAD_SHAPE;
  SkParams prm;
  prm.M = M;
  prm.N = N;
  prm.K = K;
  prm.lda = lda;
  prm.MT = (M + BM - 1) / BM;
  prm.NT = (N + bn - 1) / bn;
  prm.NKT = K / BK;
  prm.group_m = group_m;
  const long long tiles = (long long)prm.MT * prm.NT;
  if (tiles >= (1LL << 30)) return LSA_BAD_SHAPE;
  const long long iters = tiles * prm.NKT;
  prm.G = (int)(grid < iters ? grid : iters);
  prm.dp_rounds = dp ? (int)(tiles / prm.G) : 0;
  prm.sk_tiles = (int)(tiles - (long long)prm.dp_rounds * prm.G);
  prm.split = 0;
  if (epi == EPI_PARTIAL) {
    // every tile split into exactly `split` K ranges, one workgroup each, partial k written to
    // out[k]: the consumer sums exactly `split` partials, so nothing may be clamped here
    if (split > prm.NKT || tiles * split > grid) return LSA_BAD_SHAPE;
    prm.G = grid;
    prm.dp_rounds = 0;
    prm.sk_tiles = (int)tiles;
    prm.split = split;
  } else if (split > 0 && prm.sk_tiles > 0 && prm.sk_tiles <= prm.G) {
    // at most NKT ranges per tile and sk_tiles * split <= G workgroups
    prm.split = split < prm.NKT ? split : prm.NKT;
    if (prm.split > prm.G / prm.sk_tiles) prm.split = prm.G / prm.sk_tiles;
  } else if (prm.sk_tiles > 0 && (long long)prm.sk_tiles * prm.NKT < prm.G) {
    if (prm.dp_rounds > 0) {  // too few stream-K iterations for the grid: fold one round in
      prm.dp_rounds -= 1;
      prm.sk_tiles += prm.G;
    } else {
      prm.G = prm.sk_tiles * prm.NKT;  // every workgroup gets >= 1 iteration
    }
  }
  if (epi != EPI_PARTIAL && prm.sk_tiles > 0 &&
      (!slab || !counters || slab_floats < 2LL * prm.G * BM * bn || n_counters < prm.sk_tiles))
    return LSA_BAD_SHAPE;
  const bf16_raw* A = static_cast<const bf16_raw*>(a);
  const bf16_raw* W = static_cast<const bf16_raw*>(wp);
#define LSA_G(E) (bm == 256 ? dispatch<256, E>(A, W, prm, *ep, slab, counters, bn, nb, stream) \
                    : dispatch<128, E>(A, W, prm, *ep, slab, counters, bn, nb, stream))
  switch (epi) {
    case EPI_STORE: return LSA_G(EPI_STORE);
    case EPI_RESID: return LSA_G(EPI_RESID);
    case EPI_QKV: return LSA_G(EPI_QKV);
    case EPI_SWIGLU: return LSA_G(EPI_SWIGLU);
    case EPI_PARTIAL: return LSA_G(EPI_PARTIAL);
    case EPI_ARGMAX: return LSA_G(EPI_ARGMAX);
    case EPI_GEGLU: return LSA_G(EPI_GEGLU);
    default: return LSA_UNSUPPORTED;
  }
#undef LSA_G
}

#ifdef LSA_GEMM_STAMPS
extern "C" int lsa_gemm_sk_set_stamps(unsigned long long* buf) {
  return hipMemcpyToSymbol(HIP_SYMBOL(g_stamps), &buf, sizeof(buf)) == hipSuccess ? LSA_OK : LSA_LAUNCH_FAILED;
}
#endif
