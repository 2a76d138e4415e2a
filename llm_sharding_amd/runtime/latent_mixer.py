"""Latent attention as a layer mixer of :class:`.stack_engine.StackEngine`: weights and forward.

``Weights`` is loaded once per owner layer and shared by every layer that uses its tensors; the cache
belongs to the layer. One forward of a row batch (any mix of sequences, prompt portions beside
single decoded tokens), between the block's input and output projections, is

    (input             x -> [query latent | key latent, rotated key part | gate])
    append             both latents normed, rotated part turned, key side into the cache
    query projection   query latent -> q                                              one GEMM
    attention          per row in the absorbed form, or for long portions expanded (below)
    (output            gated heads -> fp32)

Rows are dealt to the two attention forms by run (consecutive positions of one sequence): a run of
at least ``expand_min`` rows multiplies keys and values of its visible tokens out once and runs the
flash kernel; everything else attends over the latents themselves.

The kernels turn pairs (i, i + rot_dims / 2); where a model pairs neighbours, the rows of its projections
that make rotated parts are put in that order once (queries and keys alike: scores do not change).
"""
from __future__ import annotations

import math

import torch
import torch.nn.functional as F

from ..models.stack import LatentSpec, pad_to
from .plan import Plan


def rotation_tables(spec: LatentSpec, n: int, device) -> tuple:
    """cos, sin [n, rot_dims / 2] fp32 of p * base^(-2i / dims)."""
    i = torch.arange(spec.rot_dims // 2, dtype=torch.float64)
    ang = torch.outer(torch.arange(n, dtype=torch.float64), spec.rot_base ** (-2.0 * i / spec.rot_dims))
    return ang.cos().float().to(device).contiguous(), ang.sin().float().to(device).contiguous()


def _head_pad(w: torch.Tensor, heads: int, parts) -> torch.Tensor:
    """Rows [heads][sum of sizes] -> [heads][sum of padded sizes], zeros behind every part.
    ``parts``: [(size, padded size), ...]."""
    v = w.view(heads, sum(s for s, _ in parts), w.shape[1])
    out, o = [], 0
    for s, p in parts:
        out.append(F.pad(v[:, o:o + s], (0, 0, 0, p - s)))
        o += s
    return torch.cat(out, 1).reshape(-1, w.shape[1])


def _halves(spec: LatentSpec, t: dict) -> dict:
    """Tensors whose rotated pairs are (i, i + rot_dims / 2)."""
    if not spec.interleaved:
        return t
    n, r = spec.rot_dims, spec.rot_dim
    at = torch.tensor(list(range(0, n, 2)) + list(range(1, n, 2)) + list(range(n, r)), device=t["dkv"].device)
    uq = t["uq"].view(spec.heads, spec.dim + r, -1)
    return {**t, "dkv": torch.cat([t["dkv"][:spec.kv_rank], t["dkv"][spec.kv_rank:][at]]),
            "uq": torch.cat([uq[:, :spec.dim], uq[:, spec.dim:][:, at]], 1).reshape(t["uq"].shape)}


class Weights:
    """One owner layer's mixer tensors, laid out for the kernels (GPU) or as they are (CPU)."""

    out_bias = None

    def __init__(self, spec: LatentSpec, t: dict, gpu: bool):
        self.spec = spec
        self.gpu = gpu
        t = _halves(spec, t)
        if not gpu:
            self.raw = t
            return
        from ..ops import latent as L
        s, H = spec, spec.heads
        self.raw = None
        self.f32 = t["dq"].dtype == torch.float32
        self.parts = [("dq", t["dq"], None, None), ("dkv", t["dkv"], None, None)]
        if s.gate:
            self.parts.append(("g", _head_pad(t["g"], H, [(s.vdim, s.dvp)]), None, None))
        self.sink = (t["sink"].float() * math.log2(math.e)).contiguous() if s.sink else None
        self.uq = L.Linear(_head_pad(t["uq"], H, [(s.dim, s.dkp), (s.rot_dim, s.rp)]))
        self.out = L.Linear(_head_pad(t["o"].t().contiguous(), H, [(s.vdim, s.dvp)]).t().contiguous())
        self.gq = t["dq.norm"].float().contiguous()
        self.gk = t["dkv.norm"].float().contiguous()
        uk = _head_pad(t["uk"], H, [(s.dim, s.dkp)])             # [H dkp, kv_rank]
        uv = _head_pad(t["uv"], H, [(s.vdim, s.dvp)])
        uk, uv = (F.pad(w, (0, s.krp - s.kv_rank)).view(H, -1, s.krp) for w in (uk, uv))
        self.tuned = L.tuned_size(s) and not self.f32            # MFMA kernels of the absorbed form
        self.expand = L.expand_size(s) and self.tuned            # MFMA kernel of the expanded form
        if self.tuned:
            self.wk = L.pack_heads(uk.transpose(1, 2))           # N = latent, K = key dimension
            self.wv = L.pack_heads(uv)                           # N = value dimension, K = latent
        else:
            self.wk = uk.contiguous()                            # [H, dkp, krp]
            self.wv = uv.transpose(1, 2).contiguous()            # [H, krp, dvp]
        self.kv = L.Linear(torch.cat([uk, uv], 1).reshape(-1, s.krp), k=s.krp) if self.expand else None

    def tensors(self) -> list:
        if not self.gpu:
            return list(self.raw.values())
        ts = [self.wk, self.wv, self.gq, self.gk] + ([self.sink] if self.sink is not None else [])
        for lin in (self.uq, self.out, self.kv):
            ts += lin.tensors() if lin is not None else []
        return ts

    def scratch(self) -> dict:
        return {"cq": self.uq.k, "q": self.uq.n, "attn": self.out.k}

    def projections(self) -> list:
        return [p for p in (self.uq, self.out, self.kv) if p is not None]

    def input_parts(self) -> list:
        return self.parts

    # ------------------------------------------------------------------ GPU
    def forward(self, eng, inp, in32, col: dict, cache: tuple, state, slot, pos, rows: int, plan) -> torch.Tensor:
        """The input projection's rows -> what the output projection reads; appends to the cache."""
        from ..ops import latent as L
        s = self.spec
        cq, cache = eng.scratch_view("cq", rows, self.uq.k), cache[0]
        q, ao = eng.scratch_view("q", rows, self.uq.n), eng.scratch_view("attn", rows, self.out.k)
        cos, sin = eng.rotation(s)
        table = eng.pool.table
        a = L.make_args(s, cache, table, slot, pos, cos, sin, eng.cfg.norm_eps, sink=self.sink)
        L.append(a, rows, inp, col["dq"], col["dkv"], self.gq, self.gk, cq)
        eng.project(self.uq, cq, rows, q)
        gate = inp[:, col["g"]:] if s.gate else None
        absorb, attend, value = ((L.absorb_mfma, L.attend_mfma, L.value_mfma) if self.tuned
                                 else (L.absorb, L.attend, L.value))
        for idx, n in absorbed_chunks(plan, self):
            b = a if idx is None else L.make_args(s, cache, table, slot, pos, cos, sin, eng.cfg.norm_eps, index=idx,
                                                 sink=self.sink)
            qt, po, pm = eng.attend_scratch()
            ns = max(1, min(key_splits(plan, self), eng.ATTEND_ITEMS // n))
            absorb(b, n, q, self.wk, qt)
            attend(b, n, qt, ns, po, pm)
            value(b, n, po, pm, ns, self.wv, gate, ao)
        for g in _split(plan, self)[2]:
            lat, kv = eng.expand_scratch(s, g.tokens, self.kv.n)
            L.gather(a, g.src, g.tokens, lat)
            eng.project(self.kv, lat, g.tokens, kv)
            L.prefill(a, g.tiles, g.tiles_host, q, kv, lat, gate, ao, rows, g.tokens)
        return ao

    # ------------------------------------------------------------------ CPU
    def forward_torch(self, eng, x, cache: tuple, state, slot, pos) -> torch.Tensor:
        """The same mixer on a CPU engine (absorbed form); its cache: [pages, 64, kv_rank + rot_dim]."""
        cache = cache[0]
        s, w, H = self.spec, {k: v.float() for k, v in self.raw.items()}, self.spec.heads
        eps, dt = eng.cfg.norm_eps, eng.dtype
        cos, sin = eng.rotation(s)
        half = s.rot_dims // 2

        def rms(v, g):
            return v * torch.rsqrt(v.pow(2).mean(-1, keepdim=True) + eps) * g

        def turn(v, p):
            c, sn = cos[p], sin[p]
            if v.dim() == 3:
                c, sn = c[:, None], sn[:, None]
            u, z, rest = v[..., :half], v[..., half:2 * half], v[..., 2 * half:]
            return torch.cat([u * c - z * sn, z * c + u * sn, rest], -1)

        d = F.linear(x, w["dkv"])
        entry = torch.cat([rms(d[:, :s.kv_rank], w["dkv.norm"]), turn(d[:, s.kv_rank:], pos)], -1)
        page = eng.pool.table[slot, pos // 64].long()
        cache[page, pos % 64] = entry.to(dt)
        q = F.linear(rms(F.linear(x, w["dq"]), w["dq.norm"]), w["uq"]).view(-1, H, s.dim + s.rot_dim)
        qt = torch.cat([torch.einsum("nhd,hdk->nhk", q[..., :s.dim], w["uk"].view(H, s.dim, s.kv_rank)),
                        turn(q[..., s.dim:], pos)], -1)
        o = torch.empty((x.shape[0], H, s.kv_rank))
        for i in range(x.shape[0]):
            n = int(pos[i]) + 1
            first = max(0, n - s.window) if s.window else 0
            keys = cache[eng.pool.table[slot[i], :-(-n // 64)].long()].reshape(-1, cache.shape[-1])[first:n].float()
            score = qt[i] @ keys.t() * s.scale
            if s.sink:
                score = torch.cat([score, w["sink"][:, None]], -1)
            p = torch.softmax(score, -1)[:, :n - first]
            o[i] = p @ keys[:, :s.kv_rank]
        v = torch.einsum("nhk,hvk->nhv", o, w["uv"].view(H, s.vdim, s.kv_rank)).reshape(x.shape[0], -1)
        return F.linear(v * torch.sigmoid(F.linear(x, w["g"])) if s.gate else v, w["o"])


def first_visible(p: int, window: int) -> int:
    """The first position that a row at position p sees."""
    return max(0, p + 1 - window) if window else 0


class Group:
    """Runs expanded together: their visible tokens (cache entries to gather) and query tiles."""

    def __init__(self, runs, tile_rows: int, device, window: int = 0):
        src, tiles, kv0 = [], [], 0
        for (row0, n, slot, p0) in runs:
            base, end = first_visible(p0, window), p0 + n
            src.append(torch.stack([torch.full((end - base,), slot), torch.arange(base, end)], 1))
            for r in range(0, n, tile_rows):
                m = min(tile_rows, n - r)
                tiles.append([row0 + r, m, kv0, p0 + r, p0 + r + m - base, base, 0, 0])
            kv0 += end - base
        tiles.sort(key=lambda t: -(t[4] - (max(0, t[3] + 1 - window - t[5]) if window else 0)))
        self.tokens = kv0
        self.src = torch.cat(src).to(torch.int32).to(device)
        self.tiles_host = torch.tensor(tiles, dtype=torch.int32)
        self.tiles = self.tiles_host.to(device)


GROUP_TOKENS = 1 << 16  # expanded tokens at a time (bounds the expanded keys' and values' memory)


def _split(plan: Plan, w: Weights) -> tuple:
    """(row indices or None for all rows, their count, groups): what runs absorbed and what expanded."""
    def make():
        idx, n, long = plan.split_rows(plan.eng.expand_min) if w.expand else (None, plan.rows, [])
        if not long:
            return None, plan.rows, []
        from ..ops import latent as L
        groups, cur, tok = [], [], 0
        rows = L.prefill_tile_rows(sum(r[1] for r in long), w.spec.heads)
        for r in long:
            n_tok = r[3] + r[1] - first_visible(r[3], w.spec.window)
            if cur and tok + n_tok > GROUP_TOKENS:
                groups.append(Group(cur, rows, plan.eng.device, w.spec.window))
                cur, tok = [], 0
            cur.append(r)
            tok += n_tok
        groups.append(Group(cur, rows, plan.eng.device, w.spec.window))
        return idx, n, groups
    return plan.memo(("latent", w.spec if w.expand else None), make)


def absorbed_chunks(plan: Plan, w: Weights) -> list:
    """[(row indices or None for all rows, count)] of the absorbed form, at most ``ATTEND_ITEMS`` at a
    time (its buffers)."""
    idx, n, _ = _split(plan, w)
    cap = plan.eng.ATTEND_ITEMS
    if idx is None and n <= cap:
        return [(None, n)] if n else []
    if idx is None:
        idx = torch.arange(n, dtype=torch.int32, device=plan.eng.device)
    return [(idx[c:c + cap], min(cap, n - c)) for c in range(0, n, cap)]


def key_splits(plan: Plan, w: Weights) -> int:
    """Splits of a row's keys, so that a small batch still fills the chip."""
    if plan._ns is not None and not w.spec.window:
        return plan._ns
    return plan.eng.latent_nsplit(w.spec, _split(plan, w)[1], plan.longest)


__all__ = ["Weights", "Group", "rotation_tables"]
