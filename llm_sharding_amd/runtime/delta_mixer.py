"""The gated delta rule as a layer mixer (:class:`..models.stack.DeltaSpec`): weights and forward.

q, k, v, the step sizes and the low-rank halves of decay and output gate ride in the block's input
projection. One forward of a row batch then is

    low rank   second halves of decay and gate                                      one GEMM
    delta      convolution, unit vectors, decays, the state and its read-out, norm and gate
    output     the block's output projection

A sequence's state lives in its slot (csrc/kernels/delta.h): the recurrence takes it from there at the start
of a run and leaves it there at its end. A run that starts at position 0 starts from zero."""
from __future__ import annotations

import torch
import torch.nn.functional as F

from ..models.stack import DeltaSpec, pad_to


class Delta:
    chunk_min = 48           # rows from which a run goes chunk by chunk (bf16) instead of step by step
    CHUNK_BYTES = 256 << 20  # workspace of one group of chunks (about what the last-level cache holds)

    def __init__(self, spec: DeltaSpec, t: dict, gpu: bool):
        self.spec, self.gpu = spec, gpu
        s = spec
        self.w = {"conv": torch.cat([t[k + ".conv"] for k in "qkv"]).float().contiguous(),
                  "decay": t["A_log"].float().exp().contiguous(), "dt_bias": t["dt_bias"].float().contiguous(),
                  "norm": t["norm"].float().contiguous()}
        self.raw = None if gpu else t
        if not gpu:
            return
        from ..ops import stream as L
        ra = pad_to(s.decay_rank, 16)
        low = F.pad(torch.cat([F.pad(t["a1"], (0, 0, 0, ra - s.decay_rank)), t["g1"]]),
                    (0, 0, 0, pad_to(ra + s.gate_rank, 128) - ra - s.gate_rank))
        self.parts = [(k, t[k], None, None) for k in "qkv"] + [("low", low, None, None), ("b", t["b"], None, "f32")]
        # second halves, side by side: output gate from g1's columns, then decay logits (fp32) from a1's
        self.oz = pad_to(s.heads * s.vdim, 16)
        w2 = torch.zeros((self.oz + s.heads * s.dim, low.shape[0]), dtype=low.dtype, device=low.device)
        w2[:s.heads * s.vdim, ra:ra + s.gate_rank] = t["g2"]
        w2[self.oz:, :s.decay_rank] = t["a2"]
        self.low = L.Linear(w2)
        self.out = L.Linear(t["o"])
        self.dtype = t["q"].dtype
        from ..ops import delta as D
        self.nbytes = D.chunk_bytes(s) if self.dtype == torch.bfloat16 else 0

    def input_parts(self) -> list:
        return self.parts

    def tensors(self) -> list:
        own = list(self.raw.values()) if self.raw is not None else self.out.tensors() + self.low.tensors()
        return own + list(self.w.values())

    def scratch(self) -> dict:
        return {"attn": self.out.k, "low": self.oz, "z": (self.low.n - self.oz, torch.float32)}

    def projections(self) -> list:
        return [self.low, self.out]

    # ------------------------------------------------------------------ GPU
    def forward(self, eng, inp, in32, col: dict, cache, state: tuple, slot, pos, rows: int, plan) -> torch.Tensor:
        from ..ops import delta as D
        s = self.spec
        gate, z = eng.scratch_view("low", rows, self.oz), eng.scratch_view("z", rows, self.low.n - self.oz)
        ao = eng.scratch_view("attn", rows, self.out.k)
        eng.project(self.low, inp[:, col["low"]:], rows, gate, out32=z, col32=self.oz)

        def args(**kw):
            return D.make_args(s, self.w, state, inp, (col["q"], col["k"], col["v"]), in32, col["b"], z, gate, ao,
                               eng.cfg.norm_eps, eng.pool.table, eng.pool.pages, **kw)
        if plan.runs is None:
            D.steps(args(slot=slot, pos=pos), self.dtype, rows, keep=True)
            return ao
        single, short, groups, long = plan.memo(("delta", s if self.nbytes else None), lambda: self._runs(plan, rows, state))
        if single is not None:
            D.steps(args(runs=single), self.dtype, single.shape[0], keep=True)
        if short is not None:
            a = args(runs=short)
            D.steps(a, self.dtype, short.shape[0], keep=False)
            D.ring(a, self.dtype, short.shape[0])
        if long is not None:
            a = args(runs=long)
            ws = eng.workspace("delta", max(c.shape[0] for c, _ in groups) * s.heads * self.nbytes)
            wide = s.heads * s.vdim
            o32 = eng.workspace("delta_o", 4 * rows * wide).view(torch.float32)[:rows * wide].view(rows, wide)
            for chunks, spans in groups:
                D.chunked(a, chunks, spans, ws, self.nbytes, o32)
            D.ring(a, self.dtype, long.shape[0])
        return ao

    def _runs(self, plan, rows: int, state: tuple) -> tuple:
        """Tables of the runs of one row, of the ones that go step by step (longest first), and the groups of
        chunks and the table of those that go in chunks; None for what the batch does not have."""
        from ..ops import delta as D
        D.check_runs(torch.tensor(plan.runs, dtype=torch.int32), rows, state[0].shape[0])
        least = self.chunk_min if self.nbytes else 1 << 30
        one, more, long = [], [], []
        for r in sorted(plan.runs, key=lambda r: -r[1]):
            (one if r[1] == 1 else more if r[1] < least else long).append(r)
        groups = D.chunk_groups(long, max(1, self.CHUNK_BYTES // (self.spec.heads * self.nbytes))) if long else []
        dev = plan.eng.device
        return tuple(plan.i32(t) if t else None for t in (one, more)) + (
            [(c.to(dev), p.to(dev)) for c, p in groups], plan.i32(long) if long else None)

    # ------------------------------------------------------------------ CPU
    def forward_torch(self, eng, x, cache, state: tuple, slot, pos) -> torch.Tensor:
        """The same mixer on a CPU engine, row by row in the order of the batch."""
        s, w = self.spec, {k: v.float() for k, v in self.raw.items()}
        S, ring = state
        n, H, G = x.shape[0], s.heads, s.kv_heads
        raw = torch.cat([F.linear(x, w[k]) for k in "qkv"], -1)
        z = (F.linear(F.linear(x, w["a1"]), w["a2"]) + w["dt_bias"]).view(n, H, s.dim)
        decay = torch.exp(-self.w["decay"][None, :, None] * F.softplus(z))
        beta = torch.sigmoid(F.linear(x, w["b"]))
        gate = torch.sigmoid(F.linear(F.linear(x, w["g1"]), w["g2"])).view(n, H, s.vdim)
        out = torch.empty(n, H, s.vdim)
        for i in range(n):
            p, sl = int(pos[i]), int(slot[i])
            ring[sl, p % s.taps] = raw[i]
            c = torch.zeros(s.channels)
            for j in range(min(s.taps, p + 1)):
                c += ring[sl, (p - j) % s.taps] * self.w["conv"][:, s.taps - 1 - j]
            q, k, v = F.silu(c).split([G * s.dim, G * s.dim, H * s.vdim])

            def unit(u):
                u = u.view(G, s.dim)
                return (u * torch.rsqrt(u.pow(2).sum(-1, keepdim=True) + s.unit_eps)).repeat_interleave(s.group, 0)
            q, k, v = unit(q) * s.q_scale, unit(k), v.view(H, s.vdim)
            st = (S[sl] if p else torch.zeros_like(S[sl])) * decay[i][..., None]
            u = beta[i][:, None] * (v - torch.einsum("hdv,hd->hv", st, k))
            st = st + k[..., None] * u[:, None]
            S[sl] = st
            o = torch.einsum("hdv,hd->hv", st, q)
            out[i] = o * torch.rsqrt(o.pow(2).mean(-1, keepdim=True) + eng.cfg.norm_eps) * self.w["norm"] * gate[i]
        return F.linear(out.reshape(n, -1), w["o"])


__all__ = ["Delta"]
