// Gated delta rule with one decay per head and key channel. Per head a state S [dim][vdim] (fp32):
//
//   S <- g * S (row by row);  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
//
// q, k, v are projections that pass a causal convolution over the last ``taps`` tokens per channel and
// silu; q and k become unit vectors. o is RMS-normed over vdim, weighted and gated.
//
// What a sequence carries from step to step is S and the convolution's last inputs, in a ring: the input
// at position p lies at ring[slot][p % taps][channel]. A sequence at position 0 starts from zero whatever
// its slot held before, so a freed slot needs no clearing.
#pragma once
#include "elem.h"

// Mirrored by llm_sharding_amd/ops/delta.py::DeltaArgs (ctypes) - keep the field order in sync.
struct DeltaArgs {
  const void* in;        // [rows][ldi] projections (bf16 or fp32): q at column oq, k at ok, v at ov
  const float* in32;     // [rows][ld32] fp32: step size logits at column ob, one per head
  const float* z;        // [rows][ldz] decay logits, heads x dim
  const void* gate;      // [rows][ldg] output gate logits, heads x vdim
  const float* conv;     // [channels][taps], channels = q (kv_heads x dim) | k | v (heads x vdim)
  const float* decay;    // [heads] exp(A_log)
  const float* dt_bias;  // [heads x dim]
  const float* norm;     // [vdim]
  float* state;          // [slots][heads][dk][dv]
  float* ring;           // [slots][taps][channels]
  const int* runs;       // [n][4] {row0, rows, slot, pos0}; null: run i is row i of slot / pos
  const int* slot;
  const int* pos;
  const int* table;      // page table: a row without a page is idle (paged_attn.h)
  void* out;             // [rows][ldo] heads x vdim
  int ldi, ld32, ldz, ldg, ldo;
  int oq, ok, ov, ob;
  int heads, kv_heads, dim, vdim, taps, dk, dv;
  int max_pages, n_pages;
  float q_scale, unit_eps, eps;
};

struct DeltaRun {
  int row0, n, slot, pos0;
};

// run i of the launch; n = 0: idle
LSA_DEVICE DeltaRun delta_run(const DeltaArgs& a, int i) {
  if (a.runs) return DeltaRun{a.runs[4 * i], a.runs[4 * i + 1], a.runs[4 * i + 2], a.runs[4 * i + 3]};
  DeltaRun r{i, 0, a.slot[i], a.pos[i]};
  if (r.pos0 >= 0 && r.pos0 < a.max_pages * 64) {
    const int pg = a.table[(size_t)r.slot * a.max_pages + r.pos0 / 64];
    r.n = pg >= 0 && pg < a.n_pages ? 1 : 0;
  }
  return r;
}

LSA_DEVICE float delta_silu(float x) { return x / (1.f + expf(-x)); }
LSA_DEVICE float delta_softplus(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }

// convolution and silu of channel ``ch`` (input column ``col``) at row t of the run
template <typename T>
LSA_DEVICE float delta_conv(const DeltaArgs& a, const DeltaRun& r, int t, int ch, int col, int channels) {
  const T* in = (const T*)a.in + (size_t)(r.row0 + t) * a.ldi + col;
  const float* w = a.conv + (size_t)ch * a.taps + a.taps - 1;
  float s = ld1(in) * w[0];
  const int p = r.pos0 + t;
  for (int j = 1; j < a.taps; ++j) {
    float x;
    if (j <= t) x = ld1(in - (size_t)j * a.ldi);
    else if (j <= p) x = a.ring[((size_t)r.slot * a.taps + (p - j) % a.taps) * channels + ch];
    else break;
    s = fmaf(x, w[-j], s);
  }
  return delta_silu(s);
}

// logarithm of the decay of head h's key channel d at a row
LSA_DEVICE float delta_log_decay(const DeltaArgs& a, int row, int h, int d) {
  return -a.decay[h] * delta_softplus(a.z[(size_t)row * a.ldz + h * a.dim + d] + a.dt_bias[h * a.dim + d]);
}

static inline bool bad_delta(const DeltaArgs* a) {
  return !a || !a->in || !a->in32 || !a->z || !a->conv || !a->decay || !a->dt_bias || !a->norm || !a->state || !a->ring ||
         !a->out || a->heads < 1 || a->kv_heads < 1 || a->heads % a->kv_heads || a->dim < 1 || a->vdim < 1 ||
         a->taps < 1 || a->dk < a->dim || a->dv < a->vdim || a->oq < 0 || a->ok < 0 || a->ov < 0 || a->ob < 0 ||
         a->ldi < a->oq + a->kv_heads * a->dim || a->ldi < a->ok + a->kv_heads * a->dim ||
         a->ldi < a->ov + a->heads * a->vdim || a->ld32 < a->ob + a->heads || a->ldz < a->heads * a->dim ||
         (a->gate && a->ldg < a->heads * a->vdim) || a->ldo < a->heads * a->vdim ||
         (!a->runs && (!a->slot || !a->pos || !a->table || a->max_pages < 1 || a->n_pages < 1));
}
