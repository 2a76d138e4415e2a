// Grouped-query attention over a paged cache: per-head scale, soft-capped scores, a sliding window that
// keeps the first tokens, and one output gate per head.
//
// A page holds 64 tokens of one layer. Keys lie token by token, values channel by channel:
//   k [n_pages][kv_heads][64][dkp]      v [n_pages][kv_heads][dvp][64]
// so that both are read as MFMA operands in 16-byte pieces. The 64 tokens of a value row are stored in
// the order in which the scores' accumulators hold them (att_vidx), which lets the weights go from
// the score tile straight into the value product.
#pragma once
#include "elem.h"

constexpr int ATT_PAGE = 64;

// Mirrored by llm_sharding_amd/ops/paged_attn.py::AttnArgs (ctypes) - keep the field order in sync.
struct AttnArgs {
  void* k;
  void* v;
  const int* table;     // [slots][max_pages] page of each 64-token stretch, -1: none
  const int* slot;      // [rows]
  const int* pos;       // [rows]
  const int* index;     // optional: entry i of the launch is row index[i]
  const float* hscale;  // [heads] score scale times the head's own number
  int max_pages;
  int n_pages;
  int heads, kv_heads;
  int dim, vdim, dkp, dvp;  // dkp, dvp: padded head parts (zeros behind)
  int window;               // a row sees keys less than this far back (INT_MAX: all) ..
  int keep;                 // .. and keys before this position
  float softcap;            // 0: none
};

// place of token r (0..63) in a value row
LSA_DEVICE int att_vidx(int r) { return (r & 32) | ((r & 12) << 1) | ((r & 16) >> 2) | (r & 3); }

LSA_DEVICE bool att_sees(const AttnArgs& a, int p, int key) {
  return key <= p && (p - key < a.window || key < a.keep);
}

// position of a live row, -1 for one whose slot holds no page there (an idle row of a decode graph)
LSA_DEVICE int att_pos(const AttnArgs& a, int row) {
  const int p = a.pos[row];
  if (p < 0 || p >= a.max_pages * ATT_PAGE) return -1;
  const int pg = a.table[(size_t)a.slot[row] * a.max_pages + p / ATT_PAGE];
  return pg < 0 || pg >= a.n_pages ? -1 : p;
}

LSA_DEVICE int att_page(const AttnArgs& a, int slot, int b) {
  const int pg = a.table[(size_t)slot * a.max_pages + b];
  return pg < 0 || pg >= a.n_pages ? 0 : pg;
}

// The key blocks (of one page each) that rows at positions p0..p1 see some key of: the kept ones, then
// those from the window's first on.
struct AttBlocks {
  int kept, first, n;
  LSA_DEVICE AttBlocks(const AttnArgs& a, int p0, int p1) {
    const int last = p1 / ATT_PAGE;
    kept = a.keep > 0 ? (min(a.keep, p1 + 1) - 1) / ATT_PAGE + 1 : 0;
    const int w = p0 - a.window + 1;  // oldest key in the first row's window
    first = max(kept, w > 0 ? w / ATT_PAGE : 0);
    n = kept + max(0, last - first + 1);
  }
  LSA_DEVICE int at(int i) const { return i < kept ? i : first + i - kept; }
};

// score (q . k) times the head's factor -> soft-capped
LSA_DEVICE float att_cap(float s, float cap, float icap) {
  // cap tanh(s / cap) = cap (1 - 2 / (exp(2 s / cap) + 1))
  return cap - 2.f * cap * __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(s * icap) + 1.f);  // icap = 2 log2(e) / cap
}
