"""How a layer's sublayers meet the fp32 residual stream, and the weights of one layer.

A block says what its sublayers read (``entry``: COPY, the stream itself in the projections' type, or the
gain of a norm of it) and leaves in ``eng.buf_x`` what it can of what the next block reads; its ``forward``
returns which of these buf_x then holds, or None. :class:`.stack_engine.StackEngine` fills the gaps.

* ``PostNorm``: mixer and feed-forward read the stream; each result is normed, scaled and added.
* ``Parallel``: both read one norm of the stream through ONE input projection (queries, keys, values, gates,
  router, up projection ...), and each result is added through a sigmoid gate per element: in the epilogue
  of the product that made it, where the stream's width allows, else in a join kernel, which also norms
  for the next block.
* ``Sandwich``: each sublayer reads a norm of the stream through one input projection; its result is normed
  again and added, in one kernel that also norms for the next sublayer.
* ``Hyper``: several streams; each sublayer reads a norm of a weighted sum of them, and its result and a matrix
  make every stream anew, in one kernel that also sums and norms for the next sublayer (``Sum``).

``Entry`` is what happens before a pass of layers that run several times in a row.
"""
from __future__ import annotations

import torch
import torch.nn.functional as F

from ..models.stack import (HYPER, PARALLEL, SANDWICH, AttentionSpec, DeltaSpec, LatentSpec, MlstmSpec, PairSpec, RetentionSpec,
                            pad_to)
from .attn_mixer import Attention
from .delta_mixer import Delta
from .feed_forward import feed_forward
from .latent_mixer import Weights
from .mlstm_mixer import Mlstm
from .retention_mixer import Pair, Retention

COPY = "copy"
MIXERS = {LatentSpec: Weights, AttentionSpec: Attention, DeltaSpec: Delta, RetentionSpec: Retention, MlstmSpec: Mlstm,
          PairSpec: Pair}


def _part(t: dict, prefix: str) -> dict:
    return {k[len(prefix):]: v for k, v in t.items() if k.startswith(prefix)}


class Layer:
    """One layer: its spec and the (possibly shared) weights of its sublayers."""

    def __init__(self, spec, weights):
        self.spec = spec
        self.w = weights

    @property
    def mixer(self):
        return self.w.mixer

    @property
    def mlp(self):
        return self.w.mlp


class InputProjection:
    """One product of the sublayers' input for everything they compute from it. ``parts``: [(name, weight, bias or
    None, kind)], kind None: a result in the engine's type, "gelu" / "relu2": with that activation, "f32": in fp32.
    They lie in this order; ``col`` has their first columns (of the fp32 result for the last kind). ``whole``: the
    width is a multiple of it (default: of 128, above 2048 of 256)."""

    KINDS = (None, "gelu", "relu2", "f32")

    def __init__(self, parts: list, name: str, whole: int = 0):
        from ..ops import hip
        from ..ops import stream as L
        parts = sorted(parts, key=lambda p: self.KINDS.index(p[3]))
        acts = {p[3] for p in parts} - {None, "f32"}
        if len(acts) > 1:
            raise ValueError(f"one activation per projection, not {acts}")
        self.act = {"gelu": hip.ACT_GELU, "relu2": hip.ACT_RELU2}.get(next(iter(acts), None), hip.ACT_NONE)
        self.name, self.col, self.act_from, self.col32, n = name, {}, None, None, 0
        for key, w, _, kind in parts:
            if kind in acts and self.act_from is None:
                self.act_from = n
            if kind == "f32" and self.col32 is None:
                self.col32 = n
            self.col[key] = n - (self.col32 or 0)
            n += pad_to(w.shape[0], 16)
        n = pad_to(n, whole or (128 if n <= 2048 else 256))
        dev, dt, o = parts[0][1].device, parts[0][1].dtype, 0
        win, bias = torch.zeros((n, parts[0][1].shape[1]), dtype=dt, device=dev), torch.zeros(n, device=dev)
        for _, w, b, _ in parts:
            win[o:o + w.shape[0]] = w
            if b is not None:
                bias[o:o + w.shape[0]] = b
            o += pad_to(w.shape[0], 16)
        self.lin = L.Linear(win)
        self.bias = bias if any(p[2] is not None for p in parts) else None
        self.n16 = self.lin.n if self.col32 is None else self.col32  # columns in the engine's type

    def tensors(self) -> list:
        return self.lin.tensors() + ([self.bias] if self.bias is not None else [])

    def scratch(self) -> dict:
        return {self.name: self.n16, self.name + "32": (self.lin.n - self.n16, torch.float32)}

    def __call__(self, eng, x, rows: int) -> tuple:
        """(results in the engine's type, fp32 results; None where there are none)."""
        n32 = self.lin.n - self.n16
        out = eng.scratch_view(self.name, rows, self.n16) if self.n16 else None
        out32 = eng.scratch_view(self.name + "32", rows, n32) if n32 else None
        if out is None:
            eng.project(self.lin, x, rows, out32, bias=self.bias)
        else:
            eng.project(self.lin, x, rows, out, bias=self.bias, out32=out32, col32=self.n16 if n32 else 0,
                        act_from=self.act_from, act=self.act)
        return out, out32


class PostNorm:
    entry = COPY

    def __init__(self, cfg, spec, t: dict, gpu: bool):
        def gain(n):  # norm weight times layer scale, fp32
            return ((t[f"norm{n}"].float() + cfg.norm_offset) * t[f"ls{n}"].float()).contiguous()
        self.mixer = MIXERS[type(spec.mixer)](spec.mixer, _part(t, "mix."), gpu)
        self.mlp = None if spec.mlp is None else feed_forward(spec.mlp, _part(t, "mlp."), gpu)
        self.gain1, self.gain2 = gain(1), None if spec.mlp is None else gain(2)
        self.inp = InputProjection(self.mixer.input_parts(), "inp", 128) if gpu else None

    def tensors(self) -> list:
        subs = [p for p in (self.inp, self.mixer, self.mlp) if p is not None]
        return [t for p in subs for t in p.tensors()] + [self.gain1, self.gain2]

    def scratch(self) -> list:
        return [self.inp.scratch(), self.mixer.scratch()] + ([self.mlp.scratch()] if self.mlp is not None else [])

    def projections(self) -> list:
        return [self.inp.lin] + self.mixer.projections() + (self.mlp.projections() if self.mlp is not None else [])

    def forward(self, eng, i: int, slot, pos, rows: int, plan, nxt):
        from ..ops import stream as L
        h, x, y, eps = eng.buf_h[:rows], eng.buf_x[:rows], eng.buf_y[:rows], eng.cfg.norm_eps
        inp, in32 = self.inp(eng, x, rows)
        ao = self.mixer.forward(eng, inp, in32, self.inp.col, eng.cache(i), eng.states[i], slot, pos, rows, plan)
        eng.project(self.mixer.out, ao, rows, y, bias=self.mixer.out_bias)
        L.stream_add_norm(y, self.gain1, eps, h, x, rows)
        if self.mlp is not None:
            y = self.mlp.forward(eng, x, None, None, {}, None, rows)["y"]
            L.stream_add_norm(y, self.gain2, eps, h, x, rows)
        return COPY

    def forward_torch(self, eng, i: int, x, slot, pos) -> torch.Tensor:
        def join(x, y, gain):
            return x + y * torch.rsqrt(y.pow(2).mean(-1, keepdim=True) + eng.cfg.norm_eps) * gain
        x = join(x, self.mixer.forward_torch(eng, x, eng.cache(i), eng.states[i], slot, pos), self.gain1)
        return x if self.mlp is None else join(x, self.mlp.forward_torch(x), self.gain2)


class Parallel:
    def __init__(self, cfg, spec, t: dict, gpu: bool):
        W = cfg.hidden_size
        self.mixer = MIXERS[type(spec.mixer)](spec.mixer, _part(t, "mix."), gpu)
        self.mlp = None if spec.mlp is None else feed_forward(spec.mlp, _part(t, "mlp."), gpu)
        self.entry = (t["norm1"].float().reshape(-1) + cfg.norm_offset).expand(W).contiguous()
        gates = [(f"rg{n}", t[f"rg{n}"], t[f"rg{n}.b"].float()) for n in ((1, 2) if self.mlp is not None else (1,))]
        self.gates = None if gpu else gates
        if not gpu:
            return
        # one projection of the norm for everything
        self.inp = InputProjection(self.mixer.input_parts() + [(n, w, b, None) for n, w, b in gates]
                                   + (self.mlp.input_parts() if self.mlp is not None else []), "inp")

    def tensors(self) -> list:
        own = [g for x in self.gates for g in x[1:]] if self.gates is not None else self.inp.tensors()
        return self.mixer.tensors() + (self.mlp.tensors() if self.mlp is not None else []) + own + [self.entry]

    def scratch(self) -> list:
        return [self.inp.scratch(), self.mixer.scratch()] + ([self.mlp.scratch()] if self.mlp is not None else [])

    def projections(self) -> list:
        return [self.inp.lin] + self.mixer.projections() + (self.mlp.projections() if self.mlp is not None else [])

    def forward(self, eng, i: int, slot, pos, rows: int, plan, nxt):
        from ..ops import stream as L
        x, h, eps = eng.buf_h[:rows], eng.buf_x[:rows], eng.cfg.norm_eps
        inp, in32 = self.inp(eng, h, rows)
        col = self.inp.col
        ao = self.mixer.forward(eng, inp, in32, col, eng.cache(i), eng.states[i], slot, pos, rows, plan)
        left = eng.project_gated(self.mixer.out, ao, rows, inp[:, col["rg1"]:], "y1", "first")
        if self.mlp is not None:
            left.update(self.mlp.forward(eng, h, inp, in32, col, inp[:, col["rg2"]:], rows))
        if not left:
            return None
        gain = nxt if isinstance(nxt, torch.Tensor) else None
        L.stream_join(x, rows, **left, gain=gain, eps=eps, out=h if gain is not None else None)
        return gain

    def forward_torch(self, eng, i: int, x, slot, pos) -> torch.Tensor:
        h = x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eng.cfg.norm_eps) * self.entry
        y = [self.mixer.forward_torch(eng, h, eng.cache(i), eng.states[i], slot, pos)]
        if self.mlp is not None:
            y.append(self.mlp.forward_torch(h))
        return x + sum(v * torch.sigmoid(F.linear(h, w.float(), b)) for v, (_, w, b) in zip(y, self.gates))


class Sandwich:
    def __init__(self, cfg, spec, t: dict, gpu: bool):
        def gain(n):
            return (t[n].float() + cfg.norm_offset).contiguous()
        self.mixer = MIXERS[type(spec.mixer)](spec.mixer, _part(t, "mix."), gpu)
        self.mlp = None if spec.mlp is None else feed_forward(spec.mlp, _part(t, "mlp."), gpu)
        self.entry, self.post1 = gain("norm1"), gain("norm1b")
        self.norm2, self.post2 = (gain("norm2"), gain("norm2b")) if self.mlp is not None else (None, None)
        if gpu:
            self.inp = InputProjection(self.mixer.input_parts(), "inp")
            self.ffin = InputProjection(self.mlp.input_parts(), "ffin") if self.mlp is not None else None
        self.inputs = [p for p in (self.inp, self.ffin) if p is not None] if gpu else []

    def _subs(self) -> list:
        return [self.mixer] + ([self.mlp] if self.mlp is not None else [])

    def tensors(self) -> list:
        own = [g for g in (self.entry, self.post1, self.norm2, self.post2) if g is not None]
        return own + [t for p in self.inputs + self._subs() for t in p.tensors()]

    def scratch(self) -> list:
        return [p.scratch() for p in self.inputs + self._subs()]

    def projections(self) -> list:
        return [p.lin for p in self.inputs] + [lin for p in self._subs() for lin in p.projections()]

    def forward(self, eng, i: int, slot, pos, rows: int, plan, nxt):
        from ..ops import stream as L
        x, h, y, eps = eng.buf_h[:rows], eng.buf_x[:rows], eng.buf_y[:rows], eng.cfg.norm_eps
        gain, out = (nxt, h) if isinstance(nxt, torch.Tensor) else (None, nxt.place(eng, rows) if nxt is not None else None)
        inp, in32 = self.inp(eng, h, rows)
        ao = self.mixer.forward(eng, inp, in32, self.inp.col, eng.cache(i), eng.states[i], slot, pos, rows, plan)
        eng.project(self.mixer.out, ao, rows, y, bias=self.mixer.out_bias)
        if self.mlp is None:
            L.stream_renorm(x, rows, y=y, post=self.post1, gain=gain, eps=eps, out=out)
            return nxt
        L.stream_renorm(x, rows, y=y, post=self.post1, gain=self.norm2, eps=eps, out=h)
        inp, in32 = self.ffin(eng, h, rows)
        left = self.mlp.forward(eng, h, inp, in32, self.ffin.col, None, rows)
        L.stream_renorm(x, rows, **left, post=self.post2, gain=gain, eps=eps, out=out)
        return nxt

    def forward_torch(self, eng, i: int, x, slot, pos) -> torch.Tensor:
        def norm(v, g):
            return v * torch.rsqrt(v.pow(2).mean(-1, keepdim=True) + eng.cfg.norm_eps) * g
        y = self.mixer.forward_torch(eng, norm(x, self.entry), eng.cache(i), eng.states[i], slot, pos)
        x = x + norm(y, self.post1)
        return x if self.mlp is None else x + norm(self.mlp.forward_torch(norm(x, self.norm2)), self.post2)


class Sum:
    """What a sublayer reads of several streams: a norm of their weighted sum."""

    def __init__(self, weights, gain):
        self.weights, self.gain = weights, gain  # fp32 [streams], [width]

    def read(self, eng, x, out, rows: int) -> None:
        from ..ops import stream as L
        L.stream_mix(x, rows, self.weights.numel(), read=self, eps=eng.cfg.norm_eps, out=out)

    def read_torch(self, eng, xs) -> torch.Tensor:
        u = torch.einsum("nsw,s->nw", xs, self.weights)
        return u * torch.rsqrt(u.pow(2).mean(-1, keepdim=True) + eng.cfg.norm_eps) * self.gain


class Hyper:
    """x_t <- sum_s mix[s, t] x_s + out[t] sublayer(norm(sum_s in[s] x_s)), for the mixer and the feed-forward."""

    def __init__(self, cfg, spec, t: dict, gpu: bool):
        self.mixer = MIXERS[type(spec.mixer)](spec.mixer, _part(t, "mix."), gpu)
        self.mlp = None if spec.mlp is None else feed_forward(spec.mlp, _part(t, "mlp."), gpu)

        def sub(n):  # (what it reads, [out | mix] of its streams)
            hc = {k: t[f"hc{n}.{k}"].float() for k in ("in", "out", "mix")}
            return (Sum(hc["in"].contiguous(), (t[f"norm{n}"].float() + cfg.norm_offset).contiguous()),
                    torch.cat([hc["out"], hc["mix"].reshape(-1)]).contiguous())
        self.entry, self.coef1 = sub(1)
        self.entry2, self.coef2 = sub(2) if self.mlp is not None else (None, None)
        self.inputs = []
        if gpu:
            self.inp = InputProjection(self.mixer.input_parts(), "inp")
            parts = self.mlp.input_parts() if self.mlp is not None else []
            self.ffin = InputProjection(parts, "ffin") if parts else None
            self.inputs = [p for p in (self.inp, self.ffin) if p is not None]

    def _subs(self) -> list:
        return [self.mixer] + ([self.mlp] if self.mlp is not None else [])

    def tensors(self) -> list:
        own = [self.coef1, self.entry.weights, self.entry.gain]
        if self.mlp is not None:
            own += [self.coef2, self.entry2.weights, self.entry2.gain]
        return own + [t for p in self.inputs + self._subs() for t in p.tensors()]

    def scratch(self) -> list:
        return [p.scratch() for p in self.inputs + self._subs()]

    def projections(self) -> list:
        return [p.lin for p in self.inputs] + [lin for p in self._subs() for lin in p.projections()]

    def forward(self, eng, i: int, slot, pos, rows: int, plan, nxt):
        from ..ops import stream as L
        x, h, y, eps, n = eng.buf_h[:rows], eng.buf_x[:rows], eng.buf_y[:rows], eng.cfg.norm_eps, eng.cfg.streams
        nxt = nxt if isinstance(nxt, Sum) else None
        inp, in32 = self.inp(eng, h, rows)
        ao = self.mixer.forward(eng, inp, in32, self.inp.col, eng.cache(i), eng.states[i], slot, pos, rows, plan)
        eng.project(self.mixer.out, ao, rows, y, bias=self.mixer.out_bias)
        second = self.entry2 if self.mlp is not None else nxt
        L.stream_mix(x, rows, n, coef=self.coef1, y=y, read=second, eps=eps, out=h)
        if self.mlp is not None:
            inp, in32 = self.ffin(eng, h, rows) if self.ffin is not None else (None, None)
            left = self.mlp.forward(eng, h, inp, in32, self.ffin.col if self.ffin is not None else {}, None, rows)
            L.stream_mix(x, rows, n, coef=self.coef2, **left, read=nxt, eps=eps, out=h)
        return nxt

    def forward_torch(self, eng, i: int, x, slot, pos) -> torch.Tensor:
        n = eng.cfg.streams
        xs = x.view(x.shape[0], n, -1)

        def join(coef, y):
            return torch.einsum("nsw,st->ntw", xs, coef[n:].view(n, n)) + coef[:n, None] * y[:, None]
        xs = join(self.coef1, self.mixer.forward_torch(eng, self.entry.read_torch(eng, xs), eng.cache(i), eng.states[i],
                                                       slot, pos))
        if self.mlp is not None:
            xs = join(self.coef2, self.mlp.forward_torch(self.entry2.read_torch(eng, xs)))
        return xs.reshape(x.shape)


class Entry:
    """What a pass of layers that run several times in a row starts from: x <- W_in [x; x0] + step[pass], x0 the
    embedding output. The stream's and x0's copies in the projections' type lie side by side, x0's from the start of
    the forward on."""

    def __init__(self, cfg, t: dict, gpu: bool):
        self.width, self.pad = cfg.hidden_size, pad_to(cfg.hidden_size, 128)
        self.raw = None if gpu else t
        if gpu:
            from ..ops import stream as L
            w, gap = t["loop.in"], (0, self.pad - self.width)
            self.lin = L.Linear(torch.cat([F.pad(w[:, :self.width], gap), F.pad(w[:, self.width:], gap)], 1))
            self.steps = F.pad(t["loop.step"].float(), (0, self.lin.n - self.width)).contiguous()

    def tensors(self) -> list:
        return list(self.raw.values()) if self.raw is not None else self.lin.tensors() + [self.steps]

    def scratch(self) -> list:
        return [{"loop": 2 * self.pad}]

    def place(self, eng, rows: int) -> torch.Tensor:
        """Where the stream's copy goes."""
        return eng.scratch_view("loop", rows, 2 * self.pad)[:, :self.pad]

    def keep(self, eng, x0, rows: int) -> None:
        from ..ops import stream as L
        L.cast_rows(x0, eng.scratch_view("loop", rows, 2 * self.pad)[:, self.pad:], rows)

    def forward(self, eng, rows: int, t: int, gain, have) -> torch.Tensor:
        """Replaces the stream; leaves its norm by ``gain`` in buf_x. ``have`` is self: the copy is in place."""
        from ..ops import stream as L
        x, y = eng.buf_h[:rows], eng.buf_y[:rows]
        if have is not self:
            L.cast_rows(x, self.place(eng, rows), rows)
        eng.project(self.lin, eng.scratch_view("loop", rows, 2 * self.pad), rows, y, bias=self.steps[t])
        L.stream_renorm(x, rows, y=y, gain=gain, eps=eng.cfg.norm_eps, out=eng.buf_x[:rows], add=False)
        return gain

    def forward_torch(self, x, x0, t: int) -> torch.Tensor:
        w = {k: v.float() for k, v in self.raw.items()}
        return F.linear(torch.cat([x, x0], -1), w["loop.in"]) + w["loop.step"][t]


BLOCKS = {PARALLEL: Parallel, SANDWICH: Sandwich, HYPER: Hyper}


def block(cfg, spec, t: dict, gpu: bool):
    return BLOCKS.get(spec.block, PostNorm)(cfg, spec, t, gpu)


__all__ = ["COPY", "Layer", "InputProjection", "PostNorm", "Parallel", "Sandwich", "Sum", "Hyper", "Entry", "block"]
