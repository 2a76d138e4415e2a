"""How a layer's sublayers meet the fp32 residual stream, and the weights of one layer.

A block says what its sublayers read (``entry``: COPY, the stream itself in the projections' type, or the
gain of a norm of it) and leaves in ``eng.buf_x`` what it can of what the next block reads; its ``forward``
returns which of these buf_x then holds, or None. :class:`.stack_engine.StackEngine` fills the gaps.

* ``PostNorm``: mixer and feed-forward read the stream; each result is normed, scaled and added.
* ``Parallel``: both read one norm of the stream through ONE input projection (queries, keys, values, gates,
  router, up projection ...), and each result is added through a sigmoid gate per element: in the epilogue
  of the product that made it, where the stream's width allows, else in a join kernel, which also norms
  for the next block.
"""
from __future__ import annotations

import torch
import torch.nn.functional as F

from ..models.stack import PARALLEL, AttentionSpec, DeltaSpec, LatentSpec, pad_to
from .attn_mixer import Attention
from .delta_mixer import Delta
from .feed_forward import feed_forward
from .latent_mixer import Weights

COPY = "copy"
MIXERS = {LatentSpec: Weights, AttentionSpec: Attention, DeltaSpec: Delta}


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


class PostNorm:
    entry = COPY

    def __init__(self, cfg, spec, t: dict, gpu: bool):
        def gain(n):  # norm weight times layer scale, fp32
            return ((t[f"norm{n}"].float() + cfg.norm_offset) * t[f"ls{n}"].float()).contiguous()
        self.mixer = MIXERS[type(spec.mixer)](spec.mixer, _part(t, "mix."), gpu)
        self.mlp = None if spec.mlp is None else feed_forward(spec.mlp, _part(t, "mlp."), gpu)
        self.gain1, self.gain2 = gain(1), None if spec.mlp is None else gain(2)

    def tensors(self) -> list:
        return self.mixer.tensors() + (self.mlp.tensors() if self.mlp is not None else []) + [self.gain1, self.gain2]

    def scratch(self) -> list:
        return [self.mixer.scratch()] + ([self.mlp.scratch()] if self.mlp is not None else [])

    def projections(self) -> list:
        return self.mixer.projections() + (self.mlp.projections() if self.mlp is not None else [])

    def forward(self, eng, i: int, slot, pos, rows: int, plan, nxt):
        from ..ops import stream as L
        h, x, y, eps = eng.buf_h[:rows], eng.buf_x[:rows], eng.buf_y[:rows], eng.cfg.norm_eps
        self.mixer.forward(eng, x, y, eng.k_cache[i], slot, pos, rows, plan)
        L.stream_add_norm(y, self.gain1, eps, h, x, rows)
        if self.mlp is not None:
            self.mlp.forward(eng, x, y, rows)
            L.stream_add_norm(y, self.gain2, eps, h, x, rows)
        return COPY

    def forward_torch(self, eng, i: int, x, slot, pos) -> torch.Tensor:
        def join(x, y, gain):
            return x + y * torch.rsqrt(y.pow(2).mean(-1, keepdim=True) + eng.cfg.norm_eps) * gain
        x = join(x, self.mixer.forward_torch(eng, x, eng.k_cache[i], slot, pos), self.gain1)
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
        from ..ops import stream as L
        # one projection of the norm for everything: parts in the engine's type, gelu'd ones last of them,
        # then parts in fp32
        parts = self.mixer.input_parts() + [(n, w, b, None) for n, w, b in gates]
        parts += self.mlp.input_parts() if self.mlp is not None else []
        parts.sort(key=lambda p: (None, "gelu", "f32").index(p[3]))
        self.col, self.gelu_from, self.col32, n = {}, None, None, 0
        for name, w, _, kind in parts:
            if kind == "gelu" and self.gelu_from is None:
                self.gelu_from = n
            if kind == "f32" and self.col32 is None:
                self.col32 = n
            self.col[name] = n - (self.col32 or 0)
            n += pad_to(w.shape[0], 16)
        n = pad_to(n, 128 if n <= 2048 else 256)
        dev, dt = parts[0][1].device, parts[0][1].dtype
        win, bias, o = torch.zeros((n, W), dtype=dt, device=dev), torch.zeros(n, dtype=torch.float32, device=dev), 0
        for _, w, b, _ in parts:
            win[o:o + w.shape[0]] = w
            if b is not None:
                bias[o:o + w.shape[0]] = b
            o += pad_to(w.shape[0], 16)
        self.inp, self.bias = L.Linear(win), bias
        self.n16 = self.inp.n if self.col32 is None else self.col32  # columns in the engine's type

    def tensors(self) -> list:
        own = [g for x in self.gates for g in x[1:]] if self.gates is not None else self.inp.tensors() + [self.bias]
        return self.mixer.tensors() + (self.mlp.tensors() if self.mlp is not None else []) + own + [self.entry]

    def scratch(self) -> list:
        own = {"inp": self.n16, "in32": (self.inp.n - self.n16, torch.float32)}
        return [own, self.mixer.scratch()] + ([self.mlp.scratch()] if self.mlp is not None else [])

    def projections(self) -> list:
        return [self.inp] + self.mixer.projections() + (self.mlp.projections() if self.mlp is not None else [])

    def forward(self, eng, i: int, slot, pos, rows: int, plan, nxt):
        from ..ops import stream as L
        x, h, eps = eng.buf_h[:rows], eng.buf_x[:rows], eng.cfg.norm_eps
        inp, in32 = eng.scratch_view("inp", rows, self.n16), None
        if self.col32 is not None:
            in32 = eng.scratch_view("in32", rows, self.inp.n - self.n16)
        eng.project(self.inp, h, rows, inp, bias=self.bias, out32=in32, col32=self.n16 if in32 is not None else 0,
                    gelu_from=self.gelu_from)
        ao = self.mixer.forward(eng, inp, in32, self.col, (eng.k_cache[i], eng.v_cache[i]), eng.states[i], slot, pos, rows,
                                plan)
        left = eng.project_gated(self.mixer.out, ao, rows, inp[:, self.col["rg1"]:], "y1", "first")
        if self.mlp is not None:
            left.update(self.mlp.forward(eng, h, inp, in32, self.col, inp[:, self.col["rg2"]:], rows))
        if not left:
            return None
        gain = nxt if isinstance(nxt, torch.Tensor) else None
        L.stream_join(x, rows, **left, gain=gain, eps=eps, out=h if gain is not None else None)
        return gain

    def forward_torch(self, eng, i: int, x, slot, pos) -> torch.Tensor:
        h = x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eng.cfg.norm_eps) * self.entry
        y = [self.mixer.forward_torch(eng, h, (eng.k_cache[i], eng.v_cache[i]), eng.states[i], slot, pos)]
        if self.mlp is not None:
            y.append(self.mlp.forward_torch(h))
        return x + sum(v * torch.sigmoid(F.linear(h, w.float(), b)) for v, (_, w, b) in zip(y, self.gates))


def block(cfg, spec, t: dict, gpu: bool):
    return (Parallel if spec.block == PARALLEL else PostNorm)(cfg, spec, t, gpu)


__all__ = ["COPY", "Layer", "PostNorm", "Parallel", "block"]
