"""Grouped-query attention over the paged cache as a layer mixer (:class:`..models.stack.AttentionSpec`):
weights and forward.

The projections of queries, keys, values and head gates ride in the block's input projection. One forward
of a row batch then is

    append      keys and values into the cache (not of a layer that reads another's)
    attention   runs of at least ``tile_min`` rows in query tiles, other rows one by one
    output      the block's output projection

A page holds keys token by token and values channel by channel (csrc/kernels/paged_attn.h). The CPU
engine keeps both token by token."""
from __future__ import annotations

import torch
import torch.nn.functional as F

from ..models.stack import AttentionSpec
from .latent_mixer import _head_pad


class Attention:
    tile_min = 16  # rows from which a run of consecutive positions goes out in query tiles

    def __init__(self, spec: AttentionSpec, t: dict, gpu: bool):
        self.spec, self.gpu = spec, gpu
        s = spec
        dev = t["q"].device
        temp = t["temp"].float() if s.head_temp else torch.ones(s.heads, device=dev)
        self.hscale = (temp * s.scale).contiguous()
        self.raw = None if gpu else t
        if not gpu:
            return
        from ..ops import paged_attn as A
        from ..ops import stream as L
        self.parts = []
        for name, heads, n, p in (("q", s.heads, s.dim, s.dkp), ("k", s.kv_heads, s.dim, s.dkp),
                                  ("v", s.kv_heads, s.vdim, s.dvp)):
            if name in t:
                bias = _head_pad(t[name + ".b"].float()[:, None], heads, [(n, p)])[:, 0] if s.bias else None
                self.parts.append((name, _head_pad(t[name], heads, [(n, p)]), bias, None))
        if s.head_gate:
            self.parts.append(("g", t["g"], None, None))
        self.out = L.Linear(_head_pad(t["o"].t().contiguous(), s.heads, [(s.vdim, s.dvp)]).t().contiguous())
        self.tuned = A.tuned_size(s) and t["q"].dtype == torch.bfloat16

    def input_parts(self) -> list:
        return self.parts

    def tensors(self) -> list:
        return list(self.raw.values()) if self.raw is not None else self.out.tensors() + [self.hscale]

    def scratch(self) -> dict:
        return {"attn": self.out.k}

    def projections(self) -> list:
        return [self.out]

    # ------------------------------------------------------------------ GPU
    def forward(self, eng, inp, in32, col: dict, cache: tuple, state, slot, pos, rows: int, plan) -> torch.Tensor:
        from ..ops import paged_attn as A
        s, table = self.spec, eng.pool.table
        ao = eng.scratch_view("attn", rows, self.out.k)
        a = A.make_args(s, cache, table, slot, pos, self.hscale)
        q = inp[:, col["q"]:]
        gate = inp[:, col["g"]:] if s.head_gate else None
        idx, n, long = plan.split_rows(self.tile_min) if self.tuned else (None, rows, [])
        b = a if idx is None else A.make_args(s, cache, table, slot, pos, self.hscale, index=idx)
        if s.kv_from is None and n:
            A.append(b, n, inp, col["k"], col["v"])
        if long:
            tiles = plan.memo(("tiles", self.tile_min), lambda: self._tiles(plan, long, rows, table))
            if s.kv_from is None:
                A.append_tiles(a, tiles, inp, col["k"], col["v"])
            A.tiles(a, tiles, q, gate, ao)
        if n and self.tuned:
            A.rows(b, n, q, gate, ao, self.key_splits(eng, n, plan.longest), eng.part_o, eng.part_ml)
        elif n:
            A.plain(b, n, q, gate, ao)
        return ao

    @staticmethod
    def _tiles(plan, long: list, rows: int, table) -> torch.Tensor:
        """Query tiles [row0, rows, slot, pos0] of the long runs, the ones with most keys first."""
        from ..ops import paged_attn as A
        t = [(r0 + c, min(A.TILE_ROWS, n - c), slot, p0 + c) for r0, n, slot, p0 in long for c in range(0, n, A.TILE_ROWS)]
        t.sort(key=lambda x: -x[3])
        host = torch.tensor(t, dtype=torch.int32)
        A.check_tiles(host, rows, *table.shape)
        return host.to(plan.eng.device)

    def key_splits(self, eng, entries: int, longest: int) -> int:
        """Splits of a row's keys: about one workgroup per CU, four pages each at least, at most 16 (the merge
        reads one partial sum per split)."""
        from ..ops import hip
        from ..ops import paged_attn as A
        s = self.spec
        seen = longest if not s.window else min(longest, s.window + 64 + -(-s.keep_first // 64) * 64)
        want = hip.N_CU // max(1, entries * A.head_tiles(s))
        cap = eng.part_o.numel() // max(1, entries * s.heads * s.dvp)
        return int(max(1, min(16, want, cap, -(-seen // (4 * A.PAGE)))))

    # ------------------------------------------------------------------ CPU
    def forward_torch(self, eng, x, cache: tuple, state, slot, pos) -> torch.Tensor:
        """The same mixer on a CPU engine; cache (keys [pages, 64, kv_heads, dim], values [.., vdim])."""
        s, w = self.spec, {k: v.float() for k, v in self.raw.items()}
        keys, values = cache
        n, dt = x.shape[0], eng.dtype

        def proj(name):
            return F.linear(x, w[name], w[name + ".b"] if s.bias else None)
        if s.kv_from is None:
            page = eng.pool.table[slot, pos // 64].long()
            keys[page, pos % 64] = proj("k").view(n, s.kv_heads, s.dim).to(dt)
            values[page, pos % 64] = proj("v").view(n, s.kv_heads, s.vdim).to(dt)
        q = proj("q").view(n, s.kv_heads, s.group, s.dim)
        gate = torch.sigmoid(F.linear(x, w["g"])) if s.head_gate else torch.ones(n, s.heads)
        o = torch.empty(n, s.heads, s.vdim)
        for i in range(n):
            p = int(pos[i])
            at = torch.arange(p + 1)
            if s.window:
                at = at[(p - at < s.window) | (at < s.keep_first)]
            pg = eng.pool.table[slot[i], at // 64].long()
            k, v = keys[pg, at % 64].float(), values[pg, at % 64].float()       # [seen, kv_heads, .]
            sc = torch.einsum("ghd,ngd->ghn", q[i], k) * self.hscale.view(s.kv_heads, s.group, 1)
            if s.softcap:
                sc = s.softcap * torch.tanh(sc / s.softcap)
            o[i] = torch.einsum("ghn,ngv->ghv", torch.softmax(sc, -1), v).reshape(s.heads, s.vdim)
        return F.linear((o * gate[..., None]).reshape(n, -1), w["o"])


__all__ = ["Attention"]
