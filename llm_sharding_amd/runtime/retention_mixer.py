"""Retention as a layer mixer (:class:`..models.stack.RetentionSpec`), and attention beside it on one input
(:class:`..models.stack.PairSpec`): weights and forward.

q, k, v and the gate ride in the block's input projection; one forward of a row batch is the recurrence with
everything around it (rotation, read-out norm, gate) and the block's output projection. A sequence's state lives
in its slot (csrc/kernels/retention.h); a run that starts at position 0 starts from zero.

A pair shares both projections: the two mixers' outputs lie side by side, each times its scale, and one output
projection takes them."""
from __future__ import annotations

import torch
import torch.nn.functional as F

from ..models.stack import PairSpec, RetentionSpec
from .attn_mixer import Attention, turned
from .latent_mixer import _head_pad


def split_runs(plan, rows: int, slots: int, spec, least: int) -> tuple:
    """Table of the runs that go step by step (longest first), segments of those of at least ``least`` rows (0: none),
    which go in chunks; None for what the batch does not have."""
    from ..ops import hip
    from ..ops import retention as X
    X.check_runs(torch.tensor(plan.runs, dtype=torch.int32), rows, slots)
    runs = sorted(plan.runs, key=lambda r: -r[1])
    long = [r for r in runs if least and r[1] >= least]
    short = runs[len(long):]
    if long:
        items, *rest = X.segments(spec, long, hip.N_CU)
        long = (items.to(plan.eng.device), *rest)
    return plan.i32(short) if short else None, long or None


class Retention:
    chunk_min = 48  # rows from which a run goes chunk by chunk (bf16) instead of step by step

    def __init__(self, spec: RetentionSpec, t: dict, gpu: bool, oscale: float = 1.0, alone: bool = True):
        """``oscale``: factor of the output; not ``alone``: ``out_weight`` goes into another's output projection."""
        self.spec, self.gpu, self.oscale, self.alone = spec, gpu, oscale, alone
        self.decay = torch.tensor(spec.decay, dtype=torch.float32, device=t["q"].device)
        self.raw = None if gpu else t
        self.out_bias = None
        if not gpu:
            return
        from ..ops import stream as L
        from ..ops import retention as X
        s, (dk, dv) = spec, spec.state_dims
        self.parts = [(c, _head_pad(t[c], s.heads, [(n, p)]), None, None)
                      for c, n, p in (("q", s.dim, dk), ("k", s.dim, dk), ("v", s.vdim, dv), ("g", s.vdim, dv))]
        weight = _head_pad(t["o"].t().contiguous(), s.heads, [(s.vdim, dv)]).t().contiguous()
        self.width, self.dtype, self.out_weight = weight.shape[1], t["q"].dtype, None if alone else weight
        self.chunks = self.dtype == torch.bfloat16 and X.chunk_size(s)
        if alone:
            self.out = L.Linear(weight)

    def input_parts(self) -> list:
        return self.parts

    def tensors(self) -> list:
        own = list(self.raw.values()) if self.raw is not None else self.out.tensors() if self.alone else []
        return own + [self.decay]

    def scratch(self) -> dict:
        return {"attn": self.out.k} if self.alone else {}

    def projections(self) -> list:
        return [self.out]

    # ------------------------------------------------------------------ GPU
    def forward(self, eng, inp, in32, col: dict, cache, state: tuple, slot, pos, rows: int, plan, ao=None) -> torch.Tensor:
        from ..ops import retention as X
        s = self.spec
        ao = eng.scratch_view("attn", rows, self.out.k) if ao is None else ao
        rot = eng.rotation(s.rot) + (s.rot.dims,) if s.rot is not None else None

        def args(**kw):
            return X.make_args(s, self.decay, state[0], inp, tuple(col[k] for k in "qkvg"), ao, rot, eng.cfg.norm_eps,
                               eng.pool.table, eng.pool.pages, oscale=self.oscale, **kw)
        if plan.runs is None:
            X.steps(args(slot=slot, pos=pos), self.dtype, rows)
            return ao
        short, long = plan.memo(("retention", s, self.chunks),
                                lambda: split_runs(plan, rows, state[0].shape[0], s, self.chunk_min if self.chunks else 0))
        if short is not None:
            X.steps(args(runs=short), self.dtype, short.shape[0])
        if long is not None:
            items, entries, longest, several = long
            (dk, dv), f32 = s.state_dims, torch.float32
            o32 = eng.workspace("ret_o", 4 * rows * s.heads * dv).view(f32)[:rows * s.heads * dv].view(rows, -1)
            ws = eng.workspace("ret", 4 * entries * s.heads * dk * dv).view(f32) if several else None
            X.chunked(args(runs=items), s, items, longest, several, ws, o32)
        return ao

    # ------------------------------------------------------------------ CPU
    def forward_torch(self, eng, x, cache, state: tuple, slot, pos) -> torch.Tensor:
        """The same mixer on a CPU engine, row by row in the order of the batch."""
        s, w = self.spec, {k: v.float() for k, v in self.raw.items()}
        S, n, H = state[0], x.shape[0], s.heads
        q, k, v, gate = (F.linear(x, w[c]).view(n, H, -1) for c in "qkvg")
        if s.rot is not None:
            q, k = (turned(eng, s.rot, y, pos) for y in (q, k))
        k = k * s.k_scale
        out = torch.empty(n, H, s.vdim)
        for i in range(n):
            sl = int(slot[i])
            st = (S[sl] if int(pos[i]) else torch.zeros_like(S[sl])) * self.decay[:, None, None]
            st = st + k[i][..., None] * v[i][:, None]
            S[sl] = st
            o = torch.einsum("hdv,hd->hv", st, q[i])
            out[i] = o * torch.rsqrt(o.pow(2).mean(-1, keepdim=True) + eng.cfg.norm_eps) * F.silu(gate[i])
        return F.linear(out.reshape(n, -1) * self.oscale, w["o"])


class Pair:
    MIXERS = {RetentionSpec: Retention}

    def __init__(self, spec: PairSpec, t: dict, gpu: bool):
        self.spec, self.gpu, self.out_bias = spec, gpu, None

        def part(side):
            return {k[len(side):]: v for k, v in t.items() if k.startswith(side)}
        self.left = Attention(spec.left, part("left."), gpu, oscale=spec.left_scale, alone=False)
        self.right = self.MIXERS[type(spec.right)](spec.right, part("right."), gpu, oscale=spec.right_scale, alone=False)
        self.sides = {"left": self.left, "right": self.right}
        if not gpu:
            return
        from ..ops import stream as L
        self.out = L.Linear(torch.cat([m.out_weight for m in self.sides.values()], 1))
        for m in self.sides.values():
            m.out_weight = None

    def input_parts(self) -> list:
        return [(f"{side}.{p[0]}", *p[1:]) for side, m in self.sides.items() for p in m.input_parts()]

    def tensors(self) -> list:
        return self.left.tensors() + self.right.tensors() + (self.out.tensors() if self.gpu else [])

    def scratch(self) -> dict:
        return {**self.left.scratch(), **self.right.scratch(), "attn": self.out.k}

    def projections(self) -> list:
        return [self.out]

    def forward(self, eng, inp, in32, col: dict, cache: tuple, state: tuple, slot, pos, rows: int, plan) -> torch.Tensor:
        ao, o = eng.scratch_view("attn", rows, self.out.k), 0
        for side, m in self.sides.items():
            sub = {k[len(side) + 1:]: v for k, v in col.items() if k.startswith(side)}
            m.forward(eng, inp, in32, sub, cache, state, slot, pos, rows, plan, ao=ao[:, o:o + m.width])
            o += m.width
        return ao

    def forward_torch(self, eng, x, cache: tuple, state: tuple, slot, pos) -> torch.Tensor:
        return sum(m.forward_torch(eng, x, cache, state, slot, pos) for m in self.sides.values())


__all__ = ["Retention", "Pair", "split_runs"]
