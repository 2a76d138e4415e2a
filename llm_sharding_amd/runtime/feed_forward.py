"""Feed-forwards of a layer stack: gated units, the dense gelu layer and the mixture of experts.

A feed-forward gives the block the rows it wants of the block's input projection (``input_parts``) and takes
their columns."""
from __future__ import annotations

import torch
import torch.nn.functional as F

from ..models.stack import SILU_GLU, DenseSpec, GluSpec, MoeSpec


class Glu:
    """Gate / up / down projection of a gated unit; gate and up are one product with the unit in its epilogue."""

    def __init__(self, spec: GluSpec, t: dict, gpu: bool):
        self.spec = spec
        self.raw = None if gpu else t
        if gpu:
            from ..ops import stream as L
            self.gate_up, self.down = L.Linear.glu(t["gate"], t["up"]), L.Linear(t["down"])
            self.bias = self.down_bias = None
            if spec.bias:
                self.bias = L.Linear.glu_bias(t["gate.b"].float(), t["up.b"].float())
                self.down_bias = F.pad(t["down.b"].float(), (0, self.down.n - t["down.b"].numel())).contiguous()

    def input_parts(self) -> list:
        return []

    def tensors(self) -> list:
        if self.raw is not None:
            return list(self.raw.values())
        return self.gate_up.tensors() + self.down.tensors() + ([self.bias, self.down_bias] if self.spec.bias else [])

    def scratch(self) -> dict:
        return {"act": self.down.k}

    def projections(self) -> list:
        return [self.gate_up, self.down]

    def forward(self, eng, h, inp, in32, col: dict, gate, rows: int) -> dict:
        act, y = eng.scratch_view("act", rows, self.down.k), eng.buf_y[:rows]
        eng.project(self.gate_up, h, rows, act, glu=self.spec, bias=self.bias)
        eng.project(self.down, act, rows, y, bias=self.down_bias)
        return {"y": y}

    def forward_torch(self, x) -> torch.Tensor:
        w, s = {k: v.float() for k, v in self.raw.items()}, self.spec
        if not s.limit:
            g, u = (F.linear(x, w[k], w.get(k + ".b")) for k in ("gate", "up"))
            return F.linear((F.gelu(g, approximate="tanh") if s.gelu else F.silu(g)) * u, w["down"], w.get("down.b"))
        g = F.linear(x, w["gate"]).clamp(max=s.limit)
        u = F.linear(x, w["up"]).clamp(-s.limit, s.limit)
        return F.linear(g * torch.sigmoid(s.alpha * g) * (u + s.shift), w["down"])


class Dense:
    """W_down gelu(W_up h): the up rows ride in the block's input projection, gelu in its epilogue."""

    def __init__(self, spec: DenseSpec, t: dict, gpu: bool):
        self.spec = spec
        self.raw = None if gpu else t
        if gpu:
            from ..ops import stream as L
            self.down = L.Linear(t["down"])
            self.up = F.pad(t["up"], (0, 0, 0, self.down.k - spec.ff))  # as wide as the down projection reads

    def input_parts(self) -> list:
        return [("up", self.up, None, "gelu")]

    def tensors(self) -> list:
        return list(self.raw.values()) if self.raw is not None else self.down.tensors()

    def scratch(self) -> dict:
        return {}

    def projections(self) -> list:
        return [self.down]

    def forward(self, eng, h, inp, in32, col: dict, gate, rows: int) -> dict:
        """The gated result joins the stream here, or is handed to the block's join."""
        act = inp[:, col["up"]:col["up"] + self.down.k]
        return eng.project_gated(self.down, act, rows, gate, "y2", "second")

    def forward_torch(self, x) -> torch.Tensor:
        w = {k: v.float() for k, v in self.raw.items()}
        return F.linear(F.gelu(F.linear(x, w["up"]), approximate="tanh"), w["down"])


class Moe:
    """Experts: routing, grouping and both products (csrc/kernels/moe.h); the router's rows, the shared expert's gate
    and, where it is no gated unit, its up rows ride in the block's input projection, the weighted sum of a row's
    experts is left to its join."""

    def __init__(self, spec: MoeSpec, t: dict, gpu: bool):
        self.spec = spec
        self.raw = None if gpu else t
        if gpu:
            from ..ops import moe as X
            from ..ops import stream as L
            e = range(spec.experts)
            self.router, self.bias = t["router"], t["router.b"].float() if spec.bias else None
            self.gate = t["shared.sg"] if spec.shared_gate else None
            gates = [t[f"e{i}.gate"] for i in e] if spec.act == SILU_GLU else None
            self.experts = X.Experts(gates, *([t[f"e{i}.{k}"] for i in e] for k in ("up", "down")))
            self.correction = t["correction"].float().contiguous() if spec.correction else None
            self.how = X.route_args(spec, self.correction)
            self.shared = self.shared_up = self.shared_glu = None
            if spec.shared_ff:
                self.shared = L.Linear(t["shared.down"])
            if spec.shared_ff and spec.act == SILU_GLU:
                self.shared_glu, self.unit = L.Linear.glu(t["shared.gate"], t["shared.up"]), GluSpec(spec.shared_ff)
            elif spec.shared_ff:
                self.shared_up = F.pad(t["shared.up"], (0, 0, 0, self.shared.k - spec.shared_ff))  # as wide as it reads

    def input_parts(self) -> list:
        own = [("shared", self.shared_up, None, "relu2")] if self.shared_up is not None else []
        own += [("sg", self.gate, None, "f32")] if self.gate is not None else []
        return own + [("router", self.router, self.bias, "f32")]

    def tensors(self) -> list:
        if self.raw is not None:
            return list(self.raw.values())
        own = [self.correction] if self.correction is not None else []
        return self.experts.tensors() + own + [t for lin in self.projections() for t in lin.tensors()]

    def scratch(self) -> dict:
        top = self.spec.top
        own = {"sact": self.shared.k} if self.shared_glu is not None else {}
        return {**own, "act": top * self.experts.ff, "ye": top * self.experts.width, "pairs": (3 * top, torch.int32),
                "tiles": (8 * top, torch.int32), "pair_w": (top, torch.float32)}

    def projections(self) -> list:
        return [lin for lin in (self.shared_glu, self.shared) if lin is not None]

    def forward(self, eng, h, inp, in32, col: dict, gate, rows: int) -> dict:
        """What the block's join adds: the experts' results, the shared one's (``y``) and the logits of its gate
        (``ygate``), and the logits of the block's gate."""
        from ..ops import moe as X
        s, x = self.spec, self.experts
        pairs = rows * s.top
        expert, order, place = eng.scratch_view("pairs", rows, 3 * s.top).reshape(3, pairs)
        weight, tiles = eng.scratch_view("pair_w", rows, s.top).reshape(-1), eng.scratch_view("tiles", rows, 8 * s.top)
        act, ye = eng.scratch_view("act", pairs, x.ff), eng.scratch_view("ye", pairs, x.width)
        tr = X.tile_rows(pairs, s.experts, x.f32)
        nt = X.route_group(in32[:, col["router"]:], rows, s.experts, s.top, tr, expert, weight, order, place, tiles,
                           self.how)
        X.gemm(tiles, nt, tr, order, s.top, h, x.up, x.up_n, x.width, act, pairs, x.kind)
        X.gemm(tiles, nt, tr, order, s.top, act, x.down, x.width, x.ff, ye, pairs, X.DOWN)
        out = {"experts": (ye, weight, place, s.top)}
        if gate is not None:
            out["gate2"] = gate
        if self.shared is not None:
            out["y"] = eng.buf_y[:rows]
            if self.shared_glu is not None:
                a = eng.scratch_view("sact", rows, self.shared.k)
                eng.project(self.shared_glu, h, rows, a, glu=self.unit)
            else:
                a = inp[:, col["shared"]:]
            eng.project(self.shared, a, rows, out["y"])
            if self.gate is not None:
                out["ygate"] = in32[:, col["sg"]:]
        return out

    def forward_torch(self, x) -> torch.Tensor:
        w, s = {k: v.float() for k, v in self.raw.items()}, self.spec
        at, weight = self._route(F.linear(x, w["router"], w.get("router.b")), w.get("correction"))

        def expert(h, name):
            up = F.linear(h, w[name + ".up"])
            a = F.silu(F.linear(h, w[name + ".gate"])) * up if s.act == SILU_GLU else F.relu(up).square()
            return F.linear(a, w[name + ".down"])
        out = expert(x, "shared") if s.shared_ff else torch.zeros_like(x)
        if s.shared_gate:
            out = out * torch.sigmoid(F.linear(x, w["shared.sg"]))
        for e in range(s.experts):
            row, k = (at == e).nonzero(as_tuple=True)
            if row.numel():
                out.index_add_(0, row, expert(x[row], f"e{e}") * weight[row, k, None])
        return out

    def _route(self, z, correction) -> tuple:
        s = self.spec
        if not s.sigmoid:
            best, at = z.topk(s.top, -1)
            return at, torch.softmax(best, -1)
        score = torch.sigmoid(z)
        choice = score + correction if s.correction else score
        if s.groups > 1:
            g = choice.view(-1, s.groups, s.experts // s.groups)
            best = g.topk(min(2, g.shape[-1]), -1).values.sum(-1).topk(s.keep, -1).indices
            ok = torch.zeros(g.shape[:2], dtype=torch.bool).scatter_(1, best, True)
            choice = g.masked_fill(~ok[..., None], float("-inf")).view_as(choice)
        at = choice.topk(s.top, -1).indices
        weight = score.gather(1, at)
        return at, weight / (weight.sum(-1, keepdim=True) + 1e-20) * s.scale


def feed_forward(spec, t: dict, gpu: bool):
    return {GluSpec: Glu, DenseSpec: Dense, MoeSpec: Moe}[type(spec)](spec, t, gpu)


__all__ = ["Glu", "Dense", "Moe", "feed_forward"]
