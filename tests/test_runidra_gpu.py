"""Runidra on the HIP path: every kernel alone against the plain equations (tests/plain_runidra.py), then the
engine: whole prompts, portions, decoding, mixed batches, reused pages and slots, generation through the
server's scheduler and captured decode graphs. fp32 engines are held to rounding; bf16 ones to what bf16
products leave."""
import json
import math
import os
import subprocess
import sys

import pytest
import torch

import plain_runidra as P
import runidra_models as M
from llm_sharding_amd.models import runidra as D
from llm_sharding_amd.models.stack import GluSpec, LatentSpec, MlstmSpec, MoeSpec
from llm_sharding_amd.parallel.server import PipelineServer

pytestmark = pytest.mark.gpu
DEV = "cuda"
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
BF, F32, F64 = torch.bfloat16, torch.float32, torch.float64
TOL = {BF: (0.025, 0.06, 0.2), F32: (4e-5,) * 3}  # engines: the median row, 49 of 50 rows, the worst row
SHARP_TOL = (1e-4,) * 3                           # fp32 engines whose softmaxes pick single keys


def _gen(seed=0):
    return torch.Generator().manual_seed(seed)


def _rand(*shape, seed=0, scale=1.0, dtype=BF):
    return (torch.randn(*shape, generator=_gen(seed)) * scale).to(dtype)


def _ids(n, vocab=150, seed=0):
    return torch.randint(0, vocab, (n,), generator=_gen(seed)).tolist()


def close(got, want, tol, what=""):
    got, want = got.double().cpu(), want.double().cpu()
    assert torch.isfinite(got).all(), what
    err = float((got - want).norm() / (want.norm() + 1e-30))
    assert err < tol, f"{what}: rel err {err:.2e} (allowed {tol:.0e})"


def rows_close(got, want, tol, what=""):
    """As :func:`close` for every row by itself: a few wrong rows do not drown among right ones."""
    got, want = got.double().cpu().flatten(1), want.double().cpu().flatten(1)
    assert torch.isfinite(got).all(), what
    err = (got - want).norm(dim=1) / (want.norm(dim=1) + 1e-30)
    assert float(err.max()) < tol, f"{what}: row {int(err.argmax())} rel err {float(err.max()):.2e} (allowed {tol:.0e})"


def held(got, want, tol, what=""):
    """Rows' differences (root mean square over the wanted rows' spread) against the limits of :data:`TOL`. In bf16 a row
    whose read-out is small before its norm, or whose router decides closely, is off by more than rounding alone: every
    kernel is held to each row above, the engines to all but a few."""
    d, w = got.double() - want.double(), want.double() - want.double().mean(-1, keepdim=True)
    e = (d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt() / w.pow(2).mean(-1).sqrt().mean()
    assert torch.isfinite(e).all(), what
    e = e.sort().values
    at = [float(e[len(e) // 2]), float(e[len(e) - 1 - len(e) // 50]), float(e[-1])]
    assert all(a < t for a, t in zip(at, tol)), f"{what}: {at} (allowed {tol})"


# ------------------------------------------------------------------------------ gated unit
@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("rows", [1, 16, 17, 40, 64, 128, 129, 300])
@pytest.mark.parametrize("ff,K", [(90, 72), (256, 200), (700, 512)])
def test_gated_gelu_with_biases(dtype, rows, ff, K):
    from llm_sharding_amd.ops import stream as L
    w = {k: _rand(*s, seed=i, scale=2 * s[-1] ** -0.5 if len(s) == 2 else 1.0) for i, (k, s) in enumerate(
        (("gate", (ff, K)), ("up", (ff, K)), ("gate.b", (ff,)), ("up.b", (ff,))))}
    x = _rand(rows, K, seed=9)
    d = {k: v.to(DEV, dtype) for k, v in w.items()}
    lin = L.Linear.glu(d["gate"], d["up"])
    xp = torch.zeros(rows, lin.k, dtype=dtype, device=DEV)
    xp[:, :K] = x.to(DEV, dtype)
    out = torch.full((rows, lin.n // 2), 7.0, dtype=dtype, device=DEV)
    g, u = (P.linear(x.double(), {k: v.double() for k, v in w.items()}, n) for n in ("gate", "up"))
    both = L.Linear.glu_bias(d["gate.b"].float(), d["up.b"].float())
    for bias, gelu in ((True, True), (False, True), (False, False)):
        lin(xp, rows, out, glu=GluSpec(ff, gelu=gelu, bias=bias), bias=both if bias else None)
        a, b = (g, u) if bias else (g - w["gate.b"].double(), u - w["up.b"].double())
        rows_close(out[:, :ff], (P.gelu(a) if gelu else P.silu(a)) * b, 1e-2 if dtype == BF else 2e-6, (bias, gelu))
        assert not out[:, ff:].any()
    with pytest.raises(ValueError):
        lin(xp, rows, out, glu=GluSpec(ff), bias=both)


# ------------------------------------------------------------------------------ streams
class Read:
    def __init__(self, weights, gain):
        self.weights, self.gain = weights.to(DEV), gain.to(DEV)


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("W", [88, 250, 4096, 9001])
@pytest.mark.parametrize("streams", [1, 2, 3, 4, 5, 16])
@pytest.mark.parametrize("rows", [5, 300])
def test_streams_mix(dtype, W, streams, rows):
    from llm_sharding_amd.ops import stream as L
    if rows > 5 and W > 4096 and streams > 3:
        rows = 260
    top, n = 3, streams
    x, y, ye = _rand(rows, n * W, seed=0, dtype=F32), _rand(rows, W, seed=1, dtype=F32), _rand(rows * top, W, seed=6)
    weight, place = torch.rand(rows * top, generator=_gen(7)), torch.randperm(rows * top, generator=_gen(8)).to(torch.int32)
    mix, out, into = _rand(n, n, seed=2, dtype=F32), _rand(n, seed=3, dtype=F32), _rand(n, seed=4, dtype=F32)
    gain, gate = _rand(W, seed=10, dtype=F32), _rand(rows, 20, seed=11, dtype=F32)
    pairs = (ye.double()[place.long()] * weight.double()[:, None]).view(rows, top, W).sum(1)
    d = {k: v.to(DEV) for k, v in dict(x=x, y=y, weight=weight, place=place, gate=gate).items()}
    coef, read = torch.cat([out, mix.flatten()]).to(DEV), Read(into, gain)
    ex = (ye.to(DEV, dtype), d["weight"], d["place"], top)
    for y_, g_, e_ in ((True, False, False), (True, True, True), (False, False, True), (True, False, True), (False, False, False)):
        xs = x.double().view(rows, n, W)
        if y_ or e_:
            v = y.double() * (torch.sigmoid(gate[:, 4:5].double()) if g_ else 1) if y_ else 0
            xs = P.scatter(xs, mix.double(), out.double(), v + (pairs if e_ else 0))
        u = P.norm(P.gather(xs, into.double()), gain.double(), 0.3)
        for read_ in (True, False):
            if not (y_ or e_ or read_):
                continue
            got, copy = d["x"].clone(), torch.full((rows, W + 4), 3.0, dtype=dtype, device=DEV)
            L.stream_mix(got, rows, n, coef=coef if y_ or e_ else None, y=d["y"] if y_ else None,
                         ygate=d["gate"][:, 4:] if g_ else None, experts=ex if e_ else None, read=read if read_ else None,
                         eps=0.3, out=copy)
            rows_close(got, xs.flatten(1), 2e-6, "streams")
            if read_:
                rows_close(copy[:, :W], u, 1e-2 if dtype == BF else 5e-6, "copy")
            assert bool((copy[:, W if read_ else 0:] == 3).all())


def test_streams_refuse_what_does_not_fit():
    from llm_sharding_amd.ops import stream as L
    x, y, read = torch.zeros(2, 64, device=DEV), torch.zeros(2, 32, device=DEV), Read(torch.ones(2), torch.ones(32))
    with pytest.raises(ValueError):
        L.stream_mix(torch.zeros(2, 17 * 32, device=DEV), 2, 17, read=read, out=y)  # more streams than it takes
    with pytest.raises(ValueError):
        L.stream_mix(x, 2, 2, coef=torch.zeros(6, device=DEV))  # nothing joins
    with pytest.raises(ValueError):
        L.stream_mix(x, 2, 2, coef=torch.zeros(5, device=DEV), y=y)


@pytest.mark.parametrize("W,streams", [(88, 3), (4096, 4), (250, 1)])
def test_embedding_fills_every_stream(W, streams):
    from llm_sharding_amd.ops import stream as L
    for dtype in (BF, F32):
        table, ids = _rand(40, W, seed=1, dtype=dtype).to(DEV), torch.tensor([3, 39, 0, 3, 7], dtype=torch.int32, device=DEV)
        x = torch.zeros(5, streams * W, device=DEV)
        L.stream_embed(ids, table, 1.5, x, None, 5, streams)
        want = (table[ids.long()].float() * 1.5)[:, None].expand(5, streams, W)
        assert torch.equal(x.view(5, streams, W), want)


def test_softcap():
    from llm_sharding_amd.ops import stream as L
    lg = _rand(7, 1501, seed=1, scale=40.0, dtype=F32).to(DEV)
    got = lg.clone()
    L.softcap_rows(got, 6, 1490, 9.0)
    rows_close(got[:6, :1490], P.capped(lg[:6, :1490].double().cpu(), 9.0), 1e-6)
    assert torch.equal(got[6], lg[6]) and torch.equal(got[:, 1490:], lg[:, 1490:])


# ------------------------------------------------------------------------------ latent attention
SIZES = {
    "small": LatentSpec(3, 20, 12, 24, 40, 33, 50.0, 12, 0.3, False, 37, True, True),
    "two_tiles": LatentSpec(20, 64, 64, 64, 64, 64, 1e4, 64, 0.2, False, 64, True, True),
    "r128": LatentSpec(33, 100, 32, 128, 128, 50, 1e4, 32, 0.2, False, 65, True, True),
    "r256": LatentSpec(16, 128, 64, 72, 200, 300, 1e3, 64, 0.15, False, 100, True, True),
    "r512": LatentSpec(32, 128, 64, 128, 512, 96, 1e4, 64, 0.15, False, 130, True, True),
    "one_key": LatentSpec(2, 16, 8, 16, 30, 20, 1e4, 8, 0.5, False, 1, True, True),
    "longer": LatentSpec(4, 32, 16, 32, 64, 40, 1e4, 16, 0.3, False, 1000, True, True),
    "no_window": LatentSpec(4, 32, 16, 32, 64, 40, 1e4, 16, 0.3, False, 0, True, True),
    "no_sink": LatentSpec(4, 32, 16, 32, 64, 40, 1e4, 16, 0.3, False, 50, False, False),
    "gated_half": LatentSpec(5, 32, 16, 40, 64, 40, 1e4, 10, 0.3, True, 50, True, True),
    "plain_wide": LatentSpec(2, 64, 32, 64, 600, 40, 1e4, 32, 0.15, False, 70, True, True),
    "plain_rot": LatentSpec(4, 32, 96, 160, 64, 40, 1e4, 96, 0.15, False, 33, True, True),
}


class LatCase:
    """A latent mixer's weights and the input rows of a few sequences, run as the engine runs it: pages that are not
    written are loud."""

    def __init__(self, s, lens, dtype, seed=0, eps=1e-3, sharp=1.0):
        from llm_sharding_amd.runtime.blocks import InputProjection
        from llm_sharding_amd.runtime.latent_mixer import Weights, rotation_tables
        self.s, self.lens, self.dtype, self.eps = s, lens, dtype, eps
        H, W = s.heads, 64
        shp = {"dq": (s.q_rank, W), "dq.norm": (s.q_rank,), "uq": (H * (s.dim + s.rot_dim), s.q_rank),
               "dkv": (s.kv_rank + s.rot_dim, W), "dkv.norm": (s.kv_rank,), "uk": (H * s.dim, s.kv_rank),
               "uv": (H * s.vdim, s.kv_rank), "o": (W, H * s.vdim)}
        if s.gate:
            shp["g"] = (H * s.vdim, W)
        self.t = {k: _rand(*v, seed=seed + i, scale=v[-1] ** -0.5 if len(v) == 2 else 1.0) for i, (k, v) in enumerate(shp.items())}
        self.t["uq"] = (self.t["uq"].float() * sharp).to(BF)
        if s.sink:
            self.t["sink"] = _rand(H, seed=99, scale=2.0)
        self.w = Weights(s, {k: v.to(DEV, dtype) for k, v in self.t.items()}, True)
        self.inp = InputProjection(self.w.input_parts(), "inp")
        self.x = [_rand(n, W, seed=seed + 30 + i) for i, n in enumerate(lens)]
        pages, self.max_pages = sum(-(-n // 64) for n in lens), max(-(-n // 64) for n in lens) + 1
        order = torch.randperm(pages, generator=_gen(seed)).tolist()
        table = torch.full((len(lens), self.max_pages), -1, dtype=torch.int32)
        for i, n in enumerate(lens):
            for b in range(-(-n // 64)):
                table[i, b] = order.pop()
        self.cache = torch.full((pages, 64, s.cache_width), 60.0, dtype=dtype, device=DEV)
        self.at, case = [0] * len(lens), self
        tables = rotation_tables(s, self.max_pages * 64, DEV)

        class Eng:  # what the mixer asks of an engine
            device, ATTEND_ITEMS, expand_min, splits = DEV, 1024, 64, None
            coop_ws = sk_ws = None

            class pool:
                pass

            class cfg:
                norm_eps = eps

            def scratch_view(self, name, rows, n):
                return torch.full((rows, n), float("nan") if name != "cq" else 0.0, dtype=dtype, device=DEV)

            def attend_scratch(self):
                def nan(n, t):
                    return torch.full((n,), float("nan"), dtype=t, device=DEV)
                return (nan(1024 * s.heads * s.cache_width, dtype), nan(1024 * s.heads * s.krp, F32), nan(1024 * s.heads * 2, F32))

            def expand_scratch(self, s, tokens, n):
                return (torch.full((tokens, s.cache_width), float("nan"), dtype=BF, device=DEV),
                        torch.full((tokens, n), float("nan"), dtype=BF, device=DEV))

            def rotation(self, s):
                return tables

            def project(self, lin, x, rows, out, glu=None, **kw):
                lin(x, rows, out, glu=glu, **kw)

            def latent_nsplit(self, s, entries, longest):
                return self.splits or 1
        self.eng = Eng()
        self.eng.pool.table = table.to(DEV)

    def want(self, i):
        s, t = self.s, {k: v.double() for k, v in self.t.items()}
        if not s.sink:
            t["sink"] = torch.full((s.heads,), -1e4, dtype=F64)
        n, H = self.lens[i], s.heads
        t["o"] = torch.eye(H * s.vdim, dtype=F64)
        m = {"heads": H, "dim": s.dim, "rot_dim": s.rot_dim, "vdim": s.vdim, "kv_rank": s.kv_rank, "scale": s.scale,
             "mask": {"size": s.window or n}, "rot": {"base": s.rot_base, "dims": s.rot_dims}}
        h = self.x[i].double()
        if not s.interleaved:  # the oracle turns neighbours
            r = s.rot_dims
            at = [j for k in range(r // 2) for j in (k, k + r // 2)] + list(range(r, s.rot_dim))
            t["dkv"] = torch.cat([t["dkv"][:s.kv_rank], t["dkv"][s.kv_rank:][at]])
            t["uq"] = torch.cat([t["uq"].view(H, -1, s.q_rank)[:, :s.dim], t["uq"].view(H, -1, s.q_rank)[:, s.dim:][:, at]],
                                1).reshape(-1, s.q_rank)
        out = P.latent_attention(h, t, m, self.eps)
        return out * torch.sigmoid(h @ t["g"].T) if s.gate else out

    def step(self, parts, splits=1):
        """One batch over the next rows of some sequences, [(sequence, rows)] -> outputs by sequence."""
        from llm_sharding_amd.runtime.plan import Plan
        s, runs, at = self.s, [], []
        for i, n in parts:
            runs.append((len(at), n, i, self.at[i]))
            at += [(i, self.at[i] + t) for t in range(n)]
            self.at[i] += n
        rows = len(at)
        slot, pos = (torch.tensor(x, dtype=torch.int32, device=DEV) for x in zip(*at))
        x = torch.zeros(rows, self.inp.lin.k, dtype=self.dtype, device=DEV)
        x[:, :64] = torch.stack([self.x[i][p] for i, p in at]).to(DEV, self.dtype)
        inp = torch.zeros(rows, self.inp.n16, dtype=self.dtype, device=DEV)
        self.inp.lin(x, rows, inp)
        self.eng.splits = splits
        out = self.w.forward(self.eng, inp, None, self.inp.col, (self.cache,), None, slot, pos, rows, Plan(self.eng, rows, runs))
        out = out[:, :s.heads * s.dvp].view(rows, s.heads, s.dvp)[..., :s.vdim].flatten(1).cpu()
        got = {}
        for (i, _), o in zip(at, out):
            got.setdefault(i, []).append(o)
        return {i: torch.stack(o) for i, o in got.items()}


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("name", list(SIZES))
def test_latent_attention(name, dtype):
    """Portions (expanded where bf16 kernels have the size), short ones and single rows of two sequences, over several
    key splits, more of them than a window has pages."""
    s = SIZES[name]
    case = LatCase(s, [330, 200], dtype)
    assert case.w.tuned == (dtype == BF and not name.startswith("plain"))
    want, got = [case.want(i) for i in (0, 1)], {0: [], 1: []}
    for parts, splits in (([(1, 1), (0, 70)], 1), ([(0, 1), (1, 66)], 3), ([(0, 130)], 1), ([(1, 2), (0, 1)], 7), ([(0, 63), (1, 64)], 2),
                          ([(0, 1)], 1), ([(0, 64), (1, 67)], 1)):
        for i, o in case.step(parts, splits).items():
            got[i].append(o)
    assert case.at == [330, 200]
    for i in (0, 1):
        rows_close(torch.cat(got[i]), want[i], 4e-2 if dtype == BF else 2e-5, f"{name}: sequence {i}")
        close(torch.cat(got[i]), want[i], 1.5e-2 if dtype == BF else 5e-6, f"{name}: sequence {i}")


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("window", [1, 7, 63, 64, 65, 100])
def test_a_key_at_the_window_edge(dtype, window):
    """A token that outweighs all others, seen by the last row of its window and not by the next: in a portion, at a
    portion's start and decoded, at page borders."""
    cfg, t = M.asking(window)
    eng = M.engine(cfg, DEV, dtype, t=t)
    for far in (0, 1, 63, 64, 65, 130):
        n = far + window + 70
        ids = _ids(n, vocab=148, seed=far)
        ids[far], ids[far + window] = M.LOUD, M.ASK
        if window > 1:
            ids[far + window - 1] = M.ASK
        want = P.run(cfg.to_dict(), t, ids)
        edge = far + window
        for cuts in ([n], [edge, n - edge], [edge - 1 or 1, 1, 1, n], [max(1, edge - 30), 31, n], [2, n]):
            eng.reset([1])
            parts, i = [], 0
            for c in cuts:
                parts.append(ids[i:i + c])
                i += len(parts[-1])
            got = torch.cat([M.feed(eng, [(1, p)]) for p in parts if p])
            held(got, want[:len(got)], TOL[dtype], (far, cuts))
        inside, outside = want[edge - 1], want[edge]
        assert window == 1 or float((inside - outside).norm() / outside.norm()) > 0.1


def test_sink_and_first_tokens():
    """The sink's share of the first rows: against the oracle, and not what a softmax without it gives."""
    s = SIZES["r128"]
    case = LatCase(s, [80], BF, sharp=0.1)
    want = case.want(0)
    sink, case.t["sink"] = case.t["sink"], torch.full((s.heads,), -1e4)
    bare = case.want(0)
    case.t["sink"] = sink
    got = torch.cat([case.step([(0, n)])[0] for n in (1, 1, 2, 76)])
    rows_close(got, want, 4e-2)
    assert float((bare[0] - want[0]).norm() / want[0].norm()) > 0.3


def test_a_sink_beyond_all_scores_and_one_below():
    for value, share in ((300.0, 0.0), (-300.0, 1.0)):
        case = LatCase(SIZES["small"], [100], BF)
        case.t["sink"].fill_(value)
        case.w.sink.fill_(value * math.log2(math.e))
        out = torch.cat([case.step([(0, n)], 3)[0] for n in (80, 3, 1, 16)])
        assert torch.isfinite(out.float()).all() and (bool(out.any()) == bool(share))
        if share:
            rows_close(out, case.want(0), 4e-2)


def test_idle_rows_leave_the_cache_alone():
    case = LatCase(SIZES["small"], [70, 70], BF)
    case.eng.pool.table[1] = -1
    before = case.cache.clone()
    out = case.step([(1, 1)])[1]
    assert not out.any() and torch.equal(before, case.cache)


# ------------------------------------------------------------------------------ matrix memory
ML = {
    "square": MlstmSpec(4, 128, 128, 15.0, 128 ** -0.5),
    "small": MlstmSpec(3, 20, 24, 6.0, 0.3),
    "wide_keys": MlstmSpec(1, 100, 32, 15.0, 0.1),
    "wide_values": MlstmSpec(2, 32, 70, 2.0, 0.2),
    "middle": MlstmSpec(2, 64, 48, 15.0, 0.125),
    "narrow": MlstmSpec(5, 48, 30, 0.5, 0.15),
    "one": MlstmSpec(1, 1, 1, 15.0, 1.0),
    "plain": MlstmSpec(2, 40, 200, 15.0, 0.15),
    "plain_keys": MlstmSpec(2, 150, 20, 15.0, 0.1),
}


class MlCase:
    """Rows of a few sequences; gates before their cap around ``bias`` +- ``spread``. A large eps: what the read-outs are
    divided by shows in spite of their norm."""

    def __init__(self, s, lens, dtype, seed=0, bias=(0.0, 2.0), spread=3.0, eps=0.05):
        self.s, self.dtype, self.lens, self.eps = s, dtype, lens, eps
        H = s.heads
        self.x = {c: [_rand(n, H, d, seed=seed + 10 * j + i) for i, n in enumerate(lens)]
                  for j, (c, d) in enumerate((("q", s.dim), ("k", s.dim), ("v", s.vdim), ("g", s.vdim)))}
        for i in range(len(lens)):  # keys lean on queries: no read-outs of almost nothing
            self.x["k"][i] = (0.5 * self.x["k"][i].float() + self.x["q"][i].float()).to(BF)
        self.z = {c: [_rand(n, H, seed=seed + 70 + 10 * j + i, scale=spread, dtype=F32) + b for i, n in enumerate(lens)]
                  for j, (c, b) in enumerate(zip("if", bias))}
        self.norm = torch.rand(H, s.vdim, generator=_gen(seed + 5)) + 0.5
        dk, dv = s.state_dims
        self.state = tuple(torch.full((len(lens), H) + shp, 3.0, device=DEV) for shp in ((dk, dv), (s.copies, dk), (s.copies,)))
        self.table = torch.zeros((len(lens), 8), dtype=torch.int32, device=DEV)
        self.norm_d = torch.nn.functional.pad(self.norm, (0, dv - s.vdim)).flatten().contiguous().to(DEV)
        self.at, self.got = [0] * len(lens), [torch.zeros(n, H, s.vdim) for n in lens]

    def want(self, i):
        s = self.s
        q, k, v, g = (self.x[c][i].double() for c in "qkvg")
        zi, zf = (P.capped(self.z[c][i].double(), s.gate_cap) for c in "if")
        out, states = torch.empty_like(v), []
        for h in range(s.heads):
            o, st = P.memory(q[:, h] * s.q_scale, k[:, h], v[:, h], zi[:, h], torch.nn.functional.logsigmoid(zf[:, h]))
            out[:, h] = P.rms(o, self.eps) * self.norm[h].double() * torch.sigmoid(g[:, h])
            states.append(st)
        return out, tuple(torch.stack(x) for x in zip(*states))

    def step(self, parts, how, wide=1):
        from llm_sharding_amd.ops import mlstm as X
        s, runs, pick = self.s, [], []
        for i, n in parts:
            runs.append((len(pick), n, i, self.at[i]))
            pick += [(i, self.at[i] + t) for t in range(n)]
            self.at[i] += n
        rows, (dk, dv), H = len(pick), s.state_dims, s.heads

        def col(c, n):
            x = torch.stack([self.x[c][i][p] for i, p in pick])
            return torch.nn.functional.pad(x, (0, n - x.shape[-1])).flatten(1)
        inp = torch.cat([torch.zeros(rows, 8, dtype=BF), col("q", dk), col("k", dk), col("v", dv), col("g", dv)], 1)
        inp = torch.nn.functional.pad(inp, (0, -inp.shape[1] % 8)).to(DEV, self.dtype)
        in32 = torch.cat([torch.stack([self.z[c][i][p] for i, p in pick]) for c in "fi"], 1).to(DEV)
        cols = (8, 8 + H * dk, 8 + 2 * H * dk, 8 + 2 * H * dk + H * dv)
        out = torch.zeros(rows, H * dv + -H * dv % 8, dtype=self.dtype, device=DEV)
        X.check_runs(torch.tensor(runs, dtype=torch.int32), rows, len(self.lens))

        def args(**kw):
            return X.make_args(s, self.norm_d, self.state, inp, in32, cols, (H, 0), out, self.eps, self.table, 8, **kw)
        if how == "rows":
            slot, pos = (torch.tensor([r[j] for r in runs], dtype=torch.int32, device=DEV) for j in (2, 3))
            X.steps(args(slot=slot, pos=pos), self.dtype, rows)
        elif how == "steps":
            X.steps(args(runs=torch.tensor(runs, dtype=torch.int32, device=DEV)), self.dtype, len(runs))
        else:
            items, entries, longest, several = X.segments(s, runs, wide, least=64)

            def nan(*n):
                return torch.full(n, float("nan"), device=DEV)
            items = items.to(DEV)
            X.chunked(args(runs=items), s, items, longest, several, nan(3 * H * rows), rows,
                      (nan(entries, H, dk, dv), nan(entries, H, s.copies, dk), nan(entries, H, s.copies, 2)), nan(rows, H * dv))
        for (i, p), o in zip(pick, out[:, :H * dv].reshape(rows, H, dv)[..., :s.vdim].cpu().float()):
            self.got[i][p] = o

    def check(self, i, what, n=None):
        n, s = self.at[i] if n is None else n, self.s
        out, (S, z, m) = self.want(i)
        tol = 6e-3 if self.dtype == BF else 2e-5
        close(self.got[i][:n], out[:n], tol, f"{what}: outputs")
        rows_close(self.got[i][:n], out[:n], 5e-2 if self.dtype == BF else 1e-3, f"{what}: outputs")
        if n == self.lens[i]:
            close(self.state[0][i, :, :s.dim, :s.vdim], S, 1e-4, f"{what}: S")
            for c in range(s.copies):
                close(self.state[1][i, :, c, :s.dim], z, 1e-4, f"{what}: n")
                assert torch.allclose(self.state[2][i, :, c].cpu().double(), m, atol=2e-5), what


@pytest.mark.parametrize("wide", [1, 1000])
@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("name", list(ML))
def test_matrix_memory(name, dtype, wide):
    """Two sequences, in step-by-step runs, single rows and (bf16) chunks and segments, all carrying the state on."""
    from llm_sharding_amd.ops import mlstm as X
    s = ML[name]
    assert X.chunk_size(s) == (not name.startswith("plain"))
    long = "chunks" if dtype == BF and X.chunk_size(s) else "steps"
    case = MlCase(s, [420, 190], dtype)
    case.step([(1, 1), (0, 1)], "rows")
    case.step([(0, 70), (1, 33)], long, wide)
    case.step([(1, 2), (0, 3)], "steps")
    for _ in range(5):
        case.step([(0, 1), (1, 1)], "rows")
    case.step([(1, 149), (0, 300)], long, wide)
    case.step([(0, 1)], "rows")
    case.step([(0, 40)], long, wide)
    assert case.at == [420, 190]
    for i in (0, 1):
        case.check(i, f"{name} {i}")
    dk, dv = s.state_dims
    rest = case.state[0].clone()
    rest[:, :, :s.dim, :s.vdim] = 0
    assert not rest.any() and not case.state[1][..., s.dim:].any()


@pytest.mark.parametrize("how,wide", [("chunks", 1), ("chunks", 1000), ("steps", 1)])
@pytest.mark.parametrize("bias,spread", [((0.0, -30.0), 1.0), ((30.0, 2.0), 1.0), ((-30.0, 30.0), 1.0), ((0.0, 0.0), 40.0), ((10.0, 6.0), 8.0)])
def test_matrix_memory_with_gates_at_their_ends(how, wide, bias, spread):
    """Forgetting all, input gates at their cap and far below, and both by turns: the running maximum follows, and large
    ones make the constant in the denominator count."""
    case = MlCase(ML["middle"], [300], BF, bias=bias, spread=spread, eps=1e-3)
    case.step([(0, 200)], how, wide)
    case.step([(0, 100)], how, wide)
    case.check(0, f"{bias} {spread}")


def test_a_portion_from_the_start_ignores_what_the_slot_held():
    for how, wide in (("steps", 1), ("chunks", 1), ("chunks", 1000), ("rows", 1)):
        case = MlCase(ML["square"], [200], BF)
        for x in case.state:
            x.fill_(1e4)
        case.step([(0, 1 if how == "rows" else 200)], how, wide)
        case.check(0, how)


def test_matrix_memory_keeps_and_forgets():
    """One loud write: the read-out three hundred rows later shows whether the head keeps it."""
    for wide in (1, 1000):
        s = MlstmSpec(2, 32, 32, 15.0, 1.0)
        case = MlCase(s, [330], BF, spread=0.0, eps=1e-6)
        for c in "qk":
            case.x[c][0][:] = 1.0
        case.x["v"][0][:] *= 0.01
        case.x["v"][0][5] = torch.arange(32) - 15.0
        case.x["g"][0][:] = 3.0
        case.z["f"][0][:, 0], case.z["f"][0][:, 1] = 12.0, -1.0
        case.step([(0, 330)], "chunks", wide)
        case.check(0, "loud")
        loud = (torch.arange(32) - 15.0) * case.norm
        for h, kept in ((0, True), (1, False)):
            o = case.got[0][329, h]
            assert (float(o @ loud[h] / o.norm() / loud[h].norm()) > 0.9) == kept


def test_idle_rows_leave_state_alone():
    from llm_sharding_amd.ops import mlstm as X
    for name in ("small", "plain"):
        case = MlCase(ML[name], [4, 4], BF)
        case.table[1] = -1
        before = [x.clone() for x in case.state]
        case.step([(1, 1)], "rows")
        assert not case.got[1].any() and all(torch.equal(a, b) for a, b in zip(before, case.state))
    with pytest.raises(ValueError):
        X.check_runs(torch.tensor([[0, 2, 0, 0], [2, 2, 0, 9]]), 4, 2)  # two runs of one slot


# ------------------------------------------------------------------------------ experts
@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("rows,experts,top,ff,shared,width", [
    (1, 8, 2, 40, 30, 72), (5, 5, 5, 130, 200, 200), (16, 6, 1, 30, 1, 64), (65, 40, 5, 20, 130, 130), (300, 4, 2, 100, 64, 144),
    (1200, 4, 2, 256, 300, 384)])
def test_experts_with_a_gated_shared_one(dtype, rows, experts, top, ff, shared, width):
    """Router biases, the softmax over the chosen, the shared expert times the sigmoid of a number per row; joined to two
    streams."""
    from llm_sharding_amd.ops import stream as L
    from llm_sharding_amd.runtime.blocks import InputProjection
    from llm_sharding_amd.runtime.feed_forward import Moe
    spec = MoeSpec(experts, top, ff, shared_ff=shared, shared_gate=True, bias=True)
    t = {k: _rand(*v, seed=i, scale=v[-1] ** -0.5 if len(v) == 2 else 3.0) for i, (k, v) in enumerate(
        D._mlp_shapes(spec, width).items())}
    t["shared.sg"] = t["shared.sg"] * 3
    moe = Moe(spec, {k: v.to(DEV, dtype) for k, v in t.items()}, True)
    x = _rand(rows, width, seed=77)
    h = torch.zeros(rows, -(-width // 128) * 128, dtype=dtype, device=DEV)
    h[:, :width] = x.to(DEV, dtype)
    flat = {}

    class Eng:
        coop_ws = sk_ws = None
        buf_y = torch.zeros(rows, h.shape[1], device=DEV)

        def scratch_view(self, name, n, k):
            if name not in flat:
                m, kind = sizes[name] if isinstance(sizes[name], tuple) else (sizes[name], dtype)
                flat[name] = torch.zeros(rows * m, dtype=kind, device=DEV)
            return flat[name][:n * k].view(n, k)

        def project(self, lin, a, n, out, glu=None, **kw):
            lin(a, n, out, glu=glu, **kw)
    inp = InputProjection(moe.input_parts(), "ffin")
    sizes = {**moe.scratch(), **inp.scratch()}
    eng = Eng()
    none, in32 = inp(eng, h, rows)
    assert none is None
    left = moe.forward(eng, h, None, in32, inp.col, None, rows)
    xs = torch.zeros(rows, 2 * width, device=DEV)
    L.stream_mix(xs, rows, 2, coef=torch.tensor([1.0, -2.0, 1.0, 0.0, 0.0, 1.0], device=DEV), **left)
    m = {"router": {"experts": experts, "top": top}}
    want = P.experts(x.double(), {k: v.double() for k, v in t.items()}, m)
    close(xs[:, :width], want, 1.2e-2 if dtype == BF else 1e-5, "experts")
    assert torch.allclose(xs[:, width:], -2 * xs[:, :width])
    if dtype == F32:
        rows_close(xs[:, :width], want, 5e-5, "experts")


# ------------------------------------------------------------------------------ engine
@pytest.fixture(scope="module")
def ordinary():
    """A model and its tensors by compute type."""
    cfg = M.stack()
    return cfg, {F32: M.tensors(cfg), BF: M.decided(cfg)}


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("sizes", [[300], [64, 1, 63, 66, 128], [2, 3, 2], [100, 65, 1, 1, 1], [1]])
def test_portions(ordinary, dtype, sizes):
    cfg, t = ordinary
    ids = _ids(300 if sizes[0] > 3 else 140)
    want = P.run(cfg.to_dict(), t[dtype], ids)
    eng = M.engine(cfg, DEV, dtype, t=t[dtype])
    got = torch.cat([M.feed(eng, [(1, p)]) for p in M.cut(ids, sizes)])
    held(got, want, TOL[dtype])


def test_streams_after_every_layer(ordinary):
    """Stages of more and more layer runs: the sum of the streams is the oracle's."""
    cfg, t = ordinary
    ids, trail = _ids(90, seed=7), []
    P.run(cfg.to_dict(), t[F32], ids, trail=trail)
    for end in range(1, cfg.num_hidden_layers + 1):
        eng = M.engine(cfg, DEV, F32, end=end)
        slot, pos = eng.prefill_rows([0], [90])
        h = eng.forward(eng.embed(torch.tensor(ids)), slot, pos)
        close(h.view(90, cfg.streams, -1).sum(1), trail[end - 1], 1e-5, f"run {end - 1}")


def test_portions_whose_softmax_picks_single_keys():
    cfg = M.stack(sharp=3.0)
    ids = _ids(330, seed=2)
    want = P.run(cfg.to_dict(), M.tensors(cfg), ids)
    for sizes in ([330], [190, 1, 2, 63], [37, 37, 3]):
        eng = M.engine(cfg, DEV, F32)
        got = torch.cat([M.feed(eng, [(0, p)]) for p in M.cut(ids, sizes)])
        held(got, want, SHARP_TOL, sizes)


@pytest.mark.parametrize("dtype", [BF, F32])
def test_long_decoding(ordinary, dtype):
    """A two-token prompt, then 330 single tokens across pages and windows."""
    cfg, t = ordinary
    ids = _ids(332, seed=5)
    want = P.run(cfg.to_dict(), t[dtype], ids)
    eng = M.engine(cfg, DEV, dtype, t=t[dtype])
    got = [M.feed(eng, [(3, ids[:2])])] + [M.feed(eng, [(3, [x])]) for x in ids[2:]]
    held(torch.cat(got), want, TOL[dtype])


@pytest.mark.parametrize("dtype", [BF, F32])
def test_unequal_batches_on_reused_pages_and_slots(ordinary, dtype):
    cfg, t = ordinary
    eng = M.engine(cfg, DEV, dtype, t=t[dtype], cache_tokens=64 * 10)
    seqs = {k: _ids(n, seed=k) for k, n in ((0, 260), (1, 75), (2, 200), (3, 140), (4, 3))}
    want = {k: P.run(cfg.to_dict(), t[dtype], v) for k, v in seqs.items()}
    slot, at, got = {0: 2, 1: 0, 2: 1, 3: 0, 4: 3}, {k: 0 for k in seqs}, {k: [] for k in seqs}

    def step(parts):
        lg = M.feed(eng, [(slot[k], seqs[k][at[k]:at[k] + n]) for k, n in parts])
        for k, n in parts:
            got[k].append(lg[:n])
            lg, at[k] = lg[n:], at[k] + n

    step([(0, 200), (1, 1)])
    step([(1, 70), (0, 1), (2, 3)])
    step([(0, 1), (2, 130), (1, 1)])
    step([(1, 3), (0, 1), (2, 1)])
    eng.reset([slot[1]])
    step([(0, 57), (2, 66), (4, 1)])
    eng.reset([slot[0], slot[2]])
    step([(3, 65), (4, 2)])
    step([(3, 75)])
    for k in seqs:
        assert at[k] == len(seqs[k])
        held(torch.cat(got[k]), want[k], TOL[dtype], k)


def test_rows_do_not_depend_on_the_batch(ordinary):
    cfg, _ = ordinary
    ids = _ids(90, seed=8)
    alone = M.engine(cfg, DEV, F32)
    M.feed(alone, [(0, ids[:89])])
    a = M.feed(alone, [(0, ids[89:])])
    other = M.engine(cfg, DEV, F32)
    M.feed(other, [(1, _ids(130, seed=3))])
    M.feed(other, [(3, ids[:50]), (0, _ids(7, seed=1))])
    M.feed(other, [(1, [4]), (3, ids[50:89])])
    b = M.feed(other, [(0, [9]), (1, [8, 7]), (3, ids[89:])])
    held(b[-1:], a, TOL[F32])


@pytest.mark.parametrize("width,streams,loop", [(130, 1, (0, 6, 2)), (144, 2, (2, 3, 1)), (129, 5, None), (64, 4, (5, 6, 3))])
def test_other_sizes_and_values_that_often_coincide(width, streams, loop):
    """Sizes beyond the tuned kernels, ones, one expert, all experts, windows of one key and of more than there are,
    scales of 1, a single stream, a whole model in the loop, a loop of one pass, none."""
    cfg = D.make_config(width, 129, [
        D.latent_entry(2, 130, 66, 200, 520, 131, 1, D.moe(1, 1, 1, 1), base=77.0),
        D.mlstm_entry(2, 140, 130, D.dense(1), 1.0),
        D.latent_entry(1, 1, 2, 1, 1, 1, 1000, D.moe(9, 9, 17, 130), scale=1.0),
        D.mlstm_entry(1, 1, 1, D.moe(8, 1, 129, 3), 50.0),
        D.latent_entry(34, 16, 64, 128, 64, 300, 64, D.dense(257), base=1e6),
        D.mlstm_entry(7, 33, 128, None)], streams, loop, eps=0.5, logit_scale=1.0 if streams == 1 else -2.0,
        logit_softcap=0.0 if streams == 2 else 2.0)
    t = M.decided(cfg)
    ids = _ids(170, vocab=129)
    want = P.run({**cfg.to_dict(), "logit_softcap": cfg.logit_softcap or 1e9}, t, ids)
    for dtype, tol in ((F32, SHARP_TOL), (BF, (0.05, 0.1, 0.3))):
        eng = M.engine(cfg, DEV, dtype, t=t)
        got = torch.cat([M.feed(eng, [(0, p)]) for p in M.cut(ids, [120, 1, 49])])
        held(got, want, tol, dtype)


def test_layers_of_a_real_width():
    """Wide heads and states, enough pairs for every expert kernel, portions on every projection kernel."""
    cfg = D.make_config(512, 260, [
        D.latent_entry(16, 128, 64, 128, 512, 256, 200, D.moe(2, 1, 256, 384)),
        D.mlstm_entry(4, 128, 128, D.moe(6, 2, 200, 100)),
        D.latent_entry(24, 64, 32, 64, 256, 128, 70, D.dense(1000))], 4, (0, 2, 2))
    t = M.decided(cfg)
    ids = _ids(850, vocab=260)
    want = P.run(cfg.to_dict(), t, ids, dtype=F32)
    eng = M.engine(cfg, DEV, BF, t=t, max_seq=1024, max_prefill_rows=1024)
    got = torch.cat([M.feed(eng, [(0, p)]) for p in M.cut(ids, [600, 1, 20, 64, 129, 2, 34])])
    held(got, want, TOL[BF])


# ------------------------------------------------------------------------------ generation
@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("graph", [True, False])
def test_greedy_generation_through_the_server(ordinary, dtype, graph):
    """More requests than slots over a small page pool, prompts cut at the prefill budget, decode graphs
    replayed while slots (and their states) come and go."""
    cfg, t = ordinary
    prompts = [_ids(n, seed=20 + n) for n in (4, 130, 1, 65, 33, 90, 7)]
    t = t[dtype]
    srv = PipelineServer(cfg, M.NamedSource(cfg, t=t), device=DEV, batch=2, microbatches=2, max_seq=192, prefill_budget=100,
                         dtype=dtype, use_graph=graph, cache_tokens=64 * 7)
    outs = srv.generate(prompts, 8, eos_ids=())
    for p, o in zip(prompts, outs):
        want, gaps = P.greedy(cfg.to_dict(), t, p, 8)
        clear = next((i for i, gp in enumerate(gaps) if gp < (0.15 if dtype == BF else 1e-3)), 8)
        assert o[:clear] == want[:clear], (len(p), o, want, gaps)
    assert len(srv.eng.pool.free) == srv.eng.pool.pages


def test_concurrent_streams_generate_the_same(ordinary):
    cfg, _ = ordinary
    prompts = [_ids(n, seed=40 + n) for n in (70, 12, 100, 5, 30, 66)]
    outs = []
    for streams in (1, 2):
        srv = PipelineServer(cfg, M.NamedSource(cfg, 0), device=DEV, batch=2, microbatches=2, max_seq=192,
                             prefill_budget=128, dtype=F32, streams=streams)
        outs.append(srv.generate(prompts, 12, eos_ids=()))
    assert outs[0] == outs[1]


@pytest.mark.parametrize("dtype", [F32, BF])
def test_graph_replays_equal_eager_steps(ordinary, dtype):
    """The capture of a graph over live sequences moves no state; replays move it as eager steps do."""
    from llm_sharding_amd.runtime.engine import DecodeGraph
    cfg, t = ordinary
    prompts = [_ids(60, seed=1), _ids(62, seed=2), _ids(3, seed=3)]
    a, b = (M.engine(cfg, DEV, dtype, t=t[dtype]) for _ in range(2))
    for eng in (a, b):
        M.feed(eng, [(i, p) for i, p in enumerate(prompts)])
    g = DecodeGraph(a, 3, "full", history_len=14)
    tok = torch.tensor([5, 6, 7], dtype=torch.int32)
    g.tokens.copy_(tok)
    g.capture()
    for i in range(14):  # crosses page and window borders
        g.replay()
        M.feed(b, [(3, [i + 1])])  # the eager engine's own work in between
        torch.cuda.synchronize()
        slot, pos = b.prefill_rows([0, 1, 2], [1, 1, 1])
        h = b.forward(b.embed(tok), slot, pos)
        b.advance([0, 1, 2], [1, 1, 1])
        assert M.rel(g.out_hidden.cpu(), h.cpu()) < (2e-2 if dtype == BF else 1e-5), i
        lg, tok = b.logits(h).cpu(), b.head(h).to(torch.int32).cpu()
        got = g.history[i].cpu()
        best = lg.max(-1).values - lg.gather(1, got.long()[:, None])[:, 0]
        assert float(best.max()) <= 2e-2 * float(lg.abs().max()), i
        g.tokens.copy_(tok)
    for s, r in zip(a.states, b.states):
        if s is not None:
            for x, y in zip(s, r):
                close(x[:3], y[:3], 2e-2 if dtype == BF else 1e-5, "state")


def test_stages_on_one_gpu():
    """Pipeline stages (split head, captured graphs, all streams between them) give the single engine's tokens."""
    from llm_sharding_amd.config import get_preset
    from llm_sharding_amd.parallel.pipeline import drive_local_pipeline, run_pipeline_generate
    cfg = get_preset("tiny-runidra")
    src = M.NamedSource(cfg, 3)
    prompts = torch.randint(3, cfg.vocab_size, (2, 2, 70), generator=_gen(4))
    kw = dict(batch=2, microbatches=2, max_seq=128, dtype=F32)
    one = run_pipeline_generate(cfg, src, prompts, 6, 0, 1, device=DEV, **kw)
    want, _ = P.greedy(cfg.to_dict(), M.tensors(cfg, 3), prompts[1, 0].tolist(), 6)
    assert one[:, 1, 0].tolist() == want
    for n in (2, 3):
        assert torch.equal(drive_local_pipeline(cfg, src, prompts, 6, n, DEV, **kw), one), n


def test_stage_costs_are_measured(ordinary):
    from llm_sharding_amd.utils.node_profiler import profile_stage_costs
    cfg, _ = ordinary
    r = profile_stage_costs(cfg, M.NamedSource(cfg, 0), DEV, batch=2, context=70, n_layers=3, prefill_len=80, replays=4)
    assert r["layer_decode_ms"] > 0 and r["layer_prefill_ms"] > 0


def test_trace_replay(ordinary, tmp_path):
    cfg, t = ordinary
    folder = D.write_random_checkpoint(cfg, str(tmp_path / "m"), seed=0)
    ids = _ids(70)
    want = P.run(cfg.to_dict(), t[F32], ids)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": ids[:66], "want": [0, 65]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": ids[:2], "want": []}, {"id": "a", "tokens": ids[66:67], "want": []}],
              "end": ["b"]},
             {"step": 2, "entries": [{"id": "c", "tokens": ids[:1], "want": [0]}, {"id": "a", "tokens": ids[67:], "want": [2]}],
              "end": ["a", "c"]}]
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", "float32",
                        "--out", str(tmp_path), "--max-tokens", "200"], input="\n".join(map(json.dumps, steps)),
                       capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 2"]

    def read(n):
        return torch.frombuffer(bytearray((tmp_path / f"{n}.f32").read_bytes()), dtype=torch.float32).view(-1, cfg.vocab_size)

    assert not (tmp_path / "1.f32").exists()
    held(read(0), want[[0, 65]], TOL[F32])
    held(read(2), want[[0, 69]], TOL[F32])
