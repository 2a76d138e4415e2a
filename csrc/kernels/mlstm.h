// Matrix memory (mLSTM). Per head a state S [dim][vdim], n [dim] and a running maximum m, all fp32 and from zero:
//
//   m' = max(f + m, i);  S <- exp(f + m - m') S + exp(i - m') k v^T;  n <- the same with k alone;  m <- m'
//   o = S^T q / (max(|n . q|, exp(-m)) + 1e-6)
//
// with log gates i = cap tanh(. / cap) and f = log sigmoid(cap tanh(. / cap)) of one fp32 projection each. q (times
// q_scale), k and v are projections; o is RMS-normed over vdim, weighted and multiplied by the sigmoid of a projected gate.
//
// Head parts are padded to dk and dv (zeros behind). n and m are stored ``copies`` times: a workgroup that advances one
// slice of the value channels reads and writes a copy of its own. A sequence at position 0 starts from zero whatever its
// slot held before, so a freed slot needs no clearing.
#pragma once
#include "elem.h"

// Mirrored by llm_sharding_amd/ops/mlstm.py::MlArgs (ctypes) - keep the field order in sync.
struct MlArgs {
  const void* in;     // [rows][ldi] projections: q at column oq (heads x dk), k at ok, v at ov (heads x dv), gate at og
  const float* in32;  // [rows][ldi32] input gates before their cap at column oi (heads), forget gates at of
  float* S;           // [slots][heads][dk][dv]
  float* n;           // [slots][heads][copies][dk]
  float* m;           // [slots][heads][copies]
  const float* norm;  // [heads][dv]
  const int* runs;    // [n][4] {row0, rows, slot, pos0}; null: run i is row i of slot / pos
  const int* slot;
  const int* pos;
  const int* table;   // page table: a row without a page is idle (paged_attn.h)
  void* out;          // [rows][ldo] heads x dv
  int ldi, ldi32, ldo, oq, ok, ov, og, oi, of;
  int heads, dim, vdim, dk, dv, copies;
  int max_pages, n_pages;
  float cap, q_scale, eps;
};

struct MlRun {
  int row0, n, slot, pos0;
};

// run i of the launch; n = 0: idle
LSA_DEVICE MlRun ml_run(const MlArgs& a, int i) {
  if (a.runs) return MlRun{a.runs[4 * i], a.runs[4 * i + 1], a.runs[4 * i + 2], a.runs[4 * i + 3]};
  MlRun r{i, 0, a.slot[i], a.pos[i]};
  if (r.pos0 >= 0 && r.pos0 < a.max_pages * 64) {
    const int pg = a.table[(size_t)r.slot * a.max_pages + r.pos0 / 64];
    r.n = pg >= 0 && pg < a.n_pages ? 1 : 0;
  }
  return r;
}

// log gates of one head of a row
LSA_DEVICE float ml_input_gate(const MlArgs& a, int row, int h) {
  return a.cap * tanhf(a.in32[(size_t)row * a.ldi32 + a.oi + h] / a.cap);
}
LSA_DEVICE float ml_forget_gate(const MlArgs& a, int row, int h) {
  const float z = a.cap * tanhf(a.in32[(size_t)row * a.ldi32 + a.of + h] / a.cap);
  return fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
}

// what S^T q is divided by
LSA_DEVICE float ml_denominator(float nq, float m) { return fmaxf(fabsf(nq), expf(-m)) + 1e-6f; }

static inline bool bad_ml(const MlArgs* a) {
  return !a || !a->in || !a->in32 || !a->S || !a->n || !a->m || !a->norm || !a->out || a->heads < 1 || a->dim < 1 ||
         a->vdim < 1 || a->dk < a->dim || a->dv < a->vdim || a->copies < 1 || !(a->cap > 0.f) || a->oq < 0 || a->ok < 0 ||
         a->ov < 0 || a->og < 0 || a->oi < 0 || a->of < 0 || a->ldi < a->oq + a->heads * a->dk ||
         a->ldi < a->ok + a->heads * a->dk || a->ldi < a->ov + a->heads * a->dv || a->ldi < a->og + a->heads * a->dv ||
         a->ldi32 < a->oi + a->heads || a->ldi32 < a->of + a->heads || a->ldo < a->heads * a->dv || a->max_pages < 1 ||
         (!a->runs && (!a->slot || !a->pos || !a->table || a->n_pages < 1));
}
