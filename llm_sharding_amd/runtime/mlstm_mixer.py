"""Matrix memory (mLSTM) as a layer mixer (:class:`..models.stack.MlstmSpec`): weights and forward.

q, k, v and the output gate ride in the block's input projection, the log gates in its fp32 columns; one forward of a row
batch is the recurrence with everything around it (gates, read-out norm, output gate) and the block's output projection. A
sequence's state lives in its slot (csrc/kernels/mlstm.h); a run that starts at position 0 starts from zero."""
from __future__ import annotations

import torch
import torch.nn.functional as F

from ..models.stack import MlstmSpec
from .latent_mixer import _head_pad
from .retention_mixer import split_runs


class Mlstm:
    chunk_min = 48  # rows from which a run goes chunk by chunk (bf16) instead of step by step
    out_bias = None

    def __init__(self, spec: MlstmSpec, t: dict, gpu: bool):
        self.spec, self.gpu = spec, gpu
        self.raw = None if gpu else t
        if not gpu:
            return
        from ..ops import mlstm as X
        from ..ops import stream as L
        s, H, (dk, dv) = spec, spec.heads, spec.state_dims
        self.parts = [(c, _head_pad(t[c], H, [(n, p)]), None, None)
                      for c, n, p in (("q", s.dim, dk), ("k", s.dim, dk), ("v", s.vdim, dv), ("g", s.vdim, dv))]
        self.parts += [(c, t[c], t[c + ".b"].float(), "f32") for c in ("i", "f")]
        self.norm = F.pad(t["norm"].float().view(H, s.vdim), (0, dv - s.vdim)).reshape(-1).contiguous()
        self.out = L.Linear(_head_pad(t["o"].t().contiguous(), H, [(s.vdim, dv)]).t().contiguous())
        self.dtype = t["q"].dtype
        self.chunks = self.dtype == torch.bfloat16 and X.chunk_size(s)

    def input_parts(self) -> list:
        return self.parts

    def tensors(self) -> list:
        return list(self.raw.values()) if self.raw is not None else self.out.tensors() + [self.norm]

    def scratch(self) -> dict:
        return {"attn": self.out.k}

    def projections(self) -> list:
        return [self.out]

    # ------------------------------------------------------------------ GPU
    def forward(self, eng, inp, in32, col: dict, cache, state: tuple, slot, pos, rows: int, plan) -> torch.Tensor:
        from ..ops import mlstm as X
        s = self.spec
        ao = eng.scratch_view("attn", rows, self.out.k)

        def args(**kw):
            return X.make_args(s, self.norm, state, inp, in32, tuple(col[k] for k in "qkvg"), (col["i"], col["f"]), ao,
                               eng.cfg.norm_eps, eng.pool.table, eng.pool.pages, **kw)
        if plan.runs is None:
            X.steps(args(slot=slot, pos=pos), self.dtype, rows)
            return ao
        short, long = plan.memo(("mlstm", s, self.chunks),
                                lambda: split_runs(plan, rows, state[0].shape[0], s, self.chunk_min if self.chunks else 0))
        if short is not None:
            X.steps(args(runs=short), self.dtype, short.shape[0])
        if long is not None:
            items, entries, longest, several = long
            (dk, dv), f32, H = s.state_dims, torch.float32, s.heads

            def ws(name, n):
                return eng.workspace(name, 4 * n).view(f32)[:n]
            o32, gates = ws("ml_o", rows * H * dv).view(rows, -1), ws("ml_g", 3 * H * rows)
            parts = tuple(ws(f"ml_{k}", entries * H * n) for k, n in (("S", dk * dv), ("n", s.copies * dk), ("m", 2 * s.copies))) \
                if several else None
            X.chunked(args(runs=items), s, items, longest, several, gates, rows, parts, o32)
        return ao

    # ------------------------------------------------------------------ CPU
    def forward_torch(self, eng, x, cache, state: tuple, slot, pos) -> torch.Tensor:
        """The same mixer on a CPU engine, row by row in the order of the batch."""
        s, w = self.spec, {k: v.float() for k, v in self.raw.items()}
        (S, N, M), n, H = state, x.shape[0], s.heads
        q, k, v, gate = (F.linear(x, w[c]).view(n, H, -1) for c in "qkvg")
        q = q * s.q_scale

        def capped(c):
            return s.gate_cap * torch.tanh(F.linear(x, w[c], w[c + ".b"]) / s.gate_cap)
        i, f = capped("i"), F.logsigmoid(capped("f"))
        out = torch.empty(n, H, s.vdim)
        for r in range(n):
            sl = int(slot[r])
            st, z, m = (S[sl], N[sl, :, 0], M[sl, :, 0]) if int(pos[r]) else (torch.zeros_like(S[sl]), torch.zeros(H, s.dim),
                                                                             torch.zeros(H))
            m1 = torch.maximum(f[r] + m, i[r])
            keep, add = torch.exp(f[r] + m - m1), torch.exp(i[r] - m1)
            st = st * keep[:, None, None] + (add[:, None] * k[r])[..., None] * v[r][:, None]
            z = z * keep[:, None] + add[:, None] * k[r]
            S[sl], N[sl, :, 0], M[sl, :, 0] = st, z, m1
            o = torch.einsum("hdv,hd->hv", st, q[r])
            o = o / (torch.maximum((z * q[r]).sum(-1).abs(), torch.exp(-m1)) + 1e-6)[:, None]
            out[r] = o * torch.rsqrt(o.pow(2).mean(-1, keepdim=True) + eng.cfg.norm_eps)
        return F.linear(out.reshape(n, -1) * w["norm"] * torch.sigmoid(gate.reshape(n, -1)), w["o"])


__all__ = ["Mlstm"]
