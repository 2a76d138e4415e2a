// Latent attention: every token leaves one latent vector (kv_rank values, all heads share it) and one
// rotated key part (rot_dim values, shared too) in a paged cache. Head h's key is
// [W_uk^h c | k_rot] and its value W_uv^h c.
//
// Two equivalent forms are used:
//   absorbed  q~ = W_uk^h^T q_h, score = q~ . c + q_rot . k_rot, value = W_uv^h (sum p c):
//             the cache is read once for all heads and nothing per head is ever expanded
//             (decode and short portions; latent.hip, latent_decode.hip)
//   expanded  keys and values of the visible tokens are multiplied out once per portion and an
//             ordinary flash attention runs over them (long portions; latent_prefill.hip)
//
// A row sees all keys up to its own or the last ``window`` of them; with ``sink`` the denominator has one
// more term per head, which belongs to no key.
#pragma once
#include "elem.h"

constexpr int LAT_PAGE = 64;  // tokens per cache page

// Mirrored by llm_sharding_amd/ops/latent.py::LatentArgs (ctypes) - keep the field order in sync.
struct LatentArgs {
  void* cache;         // this layer's pages [n_pages][LAT_PAGE][krp + rp]
  const int* table;    // [slots][max_pages] page of each 64-token stretch, -1: none
  const int* slot;     // [rows] cache slot of a row
  const int* pos;      // [rows] position of a row
  const int* index;    // optional: entry i of the launch is row index[i]
  const float* cos_t;  // [max_pages * LAT_PAGE][rot_dims / 2]
  const float* sin_t;
  const float* sink;   // [heads] log2 of a term in the softmax's denominator, null: none
  int max_pages;
  int n_pages;
  int window;             // keys a row sees, its own among them (0: all)
  int heads;
  int dim, rot_dim, rot_dims, vdim, kv_rank, q_rank;  // the model's sizes (rot_dims <= rot_dim)
  int dkp, rp, dvp, krp;  // padded: unrotated / rotated query part, value, latent (zeros behind)
  float scale;            // score scale
  float eps;              // of the two latent norms
};

// Keys a row sees, 0 for a row whose slot holds no pages (an idle row of a decode graph) or whose
// position lies outside its table.
LSA_DEVICE int lat_keys(const LatentArgs& a, int row) {
  const int p = a.pos[row];
  if (p < 0 || p >= a.max_pages * LAT_PAGE) return 0;
  const int pg = a.table[(size_t)a.slot[row] * a.max_pages + p / LAT_PAGE];
  return pg < 0 || pg >= a.n_pages ? 0 : p + 1;
}

// page of key block b (keys 64 b ..) of a row that lat_keys() found live
LSA_DEVICE int lat_page(const LatentArgs& a, int slot, int b) {
  const int pg = a.table[(size_t)slot * a.max_pages + b];
  return pg < 0 || pg >= a.n_pages ? 0 : pg;
}

// first key of a row that sees ``len`` keys without a window
LSA_DEVICE int lat_first(const LatentArgs& a, int len) { return a.window > 0 && len > a.window ? len - a.window : 0; }

// the sink's part of a denominator whose terms are 2^(score - m) (m finite: of a row that sees a key)
LSA_DEVICE float lat_sink(const LatentArgs& a, int head, float m) {
  return a.sink ? __builtin_amdgcn_exp2f(a.sink[head] - m) : 0.f;
}

// entry i of a rotated vector v (rot_dim values) at position p
template <typename T>
LSA_DEVICE float lat_rot(const LatentArgs& a, const T* v, int i, int p) {
  if (i >= a.rot_dims) return ld1(v + i);
  const int half = a.rot_dims >> 1;
  const int f = i < half ? i : i - half;
  const float c = a.cos_t[(size_t)p * half + f], s = a.sin_t[(size_t)p * half + f];
  const float u = ld1(v + f), w = ld1(v + f + half);
  return i < half ? u * c - w * s : w * c + u * s;
}
