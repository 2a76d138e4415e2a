"""Deretar on the HIP path: every kernel alone against the plain equations (tests/plain_deretar.py),
then the engine: whole prompts, portions, decoding, mixed batches, reused pages, generation through
the server's scheduler and captured decode graphs. fp32 engines are held to rounding; bf16 ones to
what bf16 products leave."""
import os
import subprocess
import sys

import pytest
import torch

import deretar_models as M
import plain_deretar as P
from llm_sharding_amd.models import deretar as D
from llm_sharding_amd.models.stack import GluSpec, LatentSpec
from llm_sharding_amd.parallel.server import PipelineServer

pytestmark = pytest.mark.gpu
DEV = "cuda"
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
BF, F32 = torch.bfloat16, torch.float32
TOL = {BF: 6e-2, F32: 2e-5}     # engines, softmaxes of ordinary width
SHARP_TOL = 3e-4                # fp32 engines whose softmaxes pick single keys


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


# ------------------------------------------------------------------------------ one mechanism at a time
@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("W", [88, 250, 4096, 9001])
def test_stream_kernels(dtype, W):
    from llm_sharding_amd.ops import latent as L
    Wp, rows, V = -(-W // 128) * 128, 7, 40
    table = _rand(V, W, seed=1, dtype=dtype).to(DEV)
    ids = torch.tensor([3, 0, 39, 39, 7, 1, 2], dtype=torch.int32, device=DEV)
    x = torch.zeros(rows, W, device=DEV)
    xc = torch.zeros(rows, Wp, dtype=dtype, device=DEV)
    L.stream_embed(ids, table, 3.25, x, xc, rows)
    assert torch.equal(x, table[ids.long()].float() * 3.25) and torch.equal(xc[:, :W], x.to(dtype))
    y, w, ls = _rand(rows, Wp, seed=2, dtype=F32), _rand(W, seed=3, scale=0.3), _rand(W, seed=4)
    y[2] = 0  # eps alone under the root
    gain = ((1 + w.float()) * ls.float()).to(DEV)
    want = P.add_normed(x.double().cpu(), y[:, :W].double(), w.double(), ls.double(), 1e-3)
    L.stream_add_norm(y.to(DEV), gain, 1e-3, x, xc, rows)
    close(x, want, 1e-6, "add_norm")
    assert torch.equal(xc[:, :W], x.to(dtype)) and not xc[:, W:].any()
    L.stream_norm(x, (1 + w.float()).to(DEV), 1e-3, xc, rows)
    close(xc[:, :W], P.centred_norm(want, w.double(), 1e-3), 5e-3 if dtype == BF else 1e-6, "norm")
    L.cast_rows(x, xc, rows)
    assert torch.equal(xc[:, :W], x.to(dtype))


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("rows", [1, 16, 17, 40, 100, 128, 129, 300])
def test_projections_take_every_size(dtype, rows):
    from llm_sharding_amd.ops import latent as L
    for N, K in ((88, 72), (330, 200)):
        w, x = _rand(N, K, seed=N), _rand(rows, K, seed=K)
        lin = L.Linear(w.to(DEV, dtype))
        xp = torch.zeros(rows, lin.k, dtype=dtype, device=DEV)
        xp[:, :K] = x.to(DEV, dtype)
        out = torch.full((rows, lin.n), 7.0, device=DEV)
        lin(xp, rows, out)
        close(out[:, :N], x.double() @ w.double().T, 1e-5, "fp32 output")
        assert not out[:, N:].any()
        gate, up = _rand(N, K, seed=1, scale=0.3), _rand(N, K, seed=2, scale=0.3)
        glu = L.Linear.glu(gate.to(DEV, dtype), up.to(DEV, dtype))
        act = torch.zeros(rows, glu.n // 2, dtype=dtype, device=DEV)
        lim = 1.5
        a, b = x.double() @ gate.double().T, x.double() @ up.double().T
        assert (a > lim).any() and (b > lim).any() and (b < -lim).any() and (a < -lim).any()
        glu(xp, rows, act, glu=GluSpec(ff=N, limit=lim, alpha=1.702, shift=1.0))
        close(act[:, :N], P.clipped_glu(a, b, lim), 5e-3 if dtype == BF else 1e-5, "gated unit")


# heads, dim, rot_dim, vdim, kv_rank, q_rank, rot_dims
SIZES = {
    "small": LatentSpec(3, 20, 12, 24, 40, 33, 50.0, 8, 0.3),
    "two_tiles": LatentSpec(20, 64, 64, 64, 64, 64, 1e4, 64, 0.2),
    "r128": LatentSpec(33, 100, 32, 128, 128, 50, 1e4, 32, 0.2),
    "r256": LatentSpec(16, 128, 64, 72, 200, 300, 1e3, 64, 0.15),
    "r512": LatentSpec(32, 128, 64, 128, 512, 96, 1e4, 64, 0.15),
    "r512_many": LatentSpec(50, 48, 64, 128, 320, 96, 1e4, 64, 0.15),
    "plain_wide": LatentSpec(2, 64, 32, 64, 600, 40, 1e4, 32, 0.15),
    "plain_rot": LatentSpec(4, 32, 96, 160, 64, 40, 1e4, 96, 0.15),
}
TUNED = [n for n in SIZES if not n.startswith("plain")]


class Case:
    """Random mixer tensors, queries and a filled cache of two slots whose pages are interleaved."""

    def __init__(self, s, lens, dtype, seed=0, sharp=1.0):
        from llm_sharding_amd.runtime.latent_mixer import Weights, rotation_tables
        self.s, self.dtype, self.lens = s, dtype, lens
        H, W = s.heads, 64
        shp = {"dq": (s.q_rank, W), "dq.norm": (s.q_rank,), "uq": (H * (s.dim + s.rot_dim), s.q_rank),
               "dkv": (s.kv_rank + s.rot_dim, W), "dkv.norm": (s.kv_rank,), "uk": (H * s.dim, s.kv_rank),
               "uv": (H * s.vdim, s.kv_rank), "g": (H * s.vdim, W), "o": (W, H * s.vdim)}
        self.t = {k: _rand(*v, seed=seed + i, scale=v[-1] ** -0.5 if len(v) == 2 else 1.0) for i, (k, v) in
                  enumerate(shp.items())}
        self.w = Weights(s, {k: v.to(DEV, dtype) for k, v in self.t.items()}, True)
        n_pages = sum(-(-n // 64) for n in lens)
        self.max_pages = max(-(-n // 64) for n in lens) + 1
        order = torch.randperm(n_pages, generator=_gen(seed)).tolist()
        self.table = torch.full((len(lens), self.max_pages), -1, dtype=torch.int32)
        self.cache = torch.full((n_pages, 64, s.cache_width), 50.0, dtype=dtype)  # stale: loud if it is read
        self.c, self.kr = [], []
        for i, n in enumerate(lens):
            c = _rand(n, s.kv_rank, seed=seed + 50 + i, dtype=dtype)
            kr = _rand(n, s.rot_dim, seed=seed + 70 + i, dtype=dtype)
            self.c.append(c)
            self.kr.append(kr)
            for b in range(-(-n // 64)):
                pg = order.pop()
                self.table[i, b] = pg
                m = min(64, n - b * 64)
                self.cache[pg, :m] = 0
                self.cache[pg, :m, :s.kv_rank] = c[b * 64:b * 64 + m]
                self.cache[pg, :m, s.krp:s.krp + s.rot_dim] = kr[b * 64:b * 64 + m]
        self.cache, self.table = self.cache.to(DEV), self.table.to(DEV)
        self.cos, self.sin = rotation_tables(s, self.max_pages * 64, DEV)
        self.sharp = sharp

    def args(self, slot, pos, index=None):
        from llm_sharding_amd.ops import latent as L
        self.slot = torch.tensor(slot, dtype=torch.int32, device=DEV)
        self.pos = torch.tensor(pos, dtype=torch.int32, device=DEV)
        return L.make_args(self.s, self.cache, self.table, self.slot, self.pos, self.cos, self.sin, 1e-4, index=index)

    def queries(self, rows, seed=7):
        s = self.s
        q = _rand(rows, s.heads, s.dim + s.rot_dim, seed=seed, scale=self.sharp, dtype=self.dtype)
        pad = torch.zeros(rows, s.heads, s.dkp + s.rp, dtype=self.dtype)
        pad[..., :s.dim], pad[..., s.dkp:s.dkp + s.rot_dim] = q[..., :s.dim], q[..., s.dim:]
        return q, torch.nn.functional.pad(pad.flatten(1), (0, self.w.uq.n - s.heads * (s.dkp + s.rp))).to(DEV)

    def want(self, q, slot, pos, gate=None):
        """Heads' outputs by the plain equations, one row at a time."""
        s, H = self.s, self.s.heads
        uk, uv = self.t["uk"].double().view(H, s.dim, -1), self.t["uv"].double().view(H, s.vdim, -1)
        out = []
        for i in range(len(pos)):
            c, kr = self.c[slot[i]][:pos[i] + 1].double(), self.kr[slot[i]][:pos[i] + 1].double()
            qn = q[i, :, :s.dim].double()
            qr = P.rotate(q[i:i + 1, :, s.dim:].double(), torch.tensor([pos[i]]), s.rot_base, s.rot_dims)[0]
            sc = (torch.einsum("hd,hdk,nk->hn", qn, uk, c) + qr @ kr.T) * s.scale
            p = torch.softmax(sc, -1)
            out.append(torch.einsum("hn,nk,hvk->hv", p, c, uv).reshape(-1))
        o = torch.stack(out)
        return o if gate is None else o * torch.sigmoid(gate.double())

    def unpad(self, out):
        s = self.s
        return out[:, :s.heads * s.dvp].view(-1, s.heads, s.dvp)[..., :s.vdim].flatten(1)


def _absorbed(case, slot, pos, q, ns, gate=None, index=None):
    from llm_sharding_amd.ops import latent as L
    s, w = case.s, case.w
    n = len(pos) if index is None else index.numel()
    a = case.args(slot, pos, index)
    qt = torch.zeros(n * s.heads * s.cache_width, dtype=case.dtype, device=DEV)
    po = torch.full((n * s.heads * ns * s.krp,), float("nan"), device=DEV)
    pm = torch.full((n * s.heads * ns * 2,), float("nan"), device=DEV)
    out = torch.zeros(len(pos), w.out.k, dtype=case.dtype, device=DEV)
    f = (L.absorb_mfma, L.attend_mfma, L.value_mfma) if w.tuned else (L.absorb, L.attend, L.value)
    f[0](a, n, q, w.wk, qt)
    f[1](a, n, qt, ns, po, pm)
    f[2](a, n, po, pm, ns, w.wv, gate, out)
    return out


def _gate(case, rows):
    s = case.s
    g = _rand(rows, s.heads, s.vdim, seed=9, dtype=case.dtype)
    pad = torch.zeros(rows, s.heads, s.dvp, dtype=case.dtype)
    pad[..., :s.vdim] = g
    return g.flatten(1), pad.flatten(1).to(DEV)


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("name", list(SIZES))
def test_absorbed_attention(name, dtype):
    """Rows of two sequences at page borders, split over 1, 3 and more splits than pages."""
    s = SIZES[name]
    case = Case(s, [200, 130], dtype)
    assert case.w.tuned == (dtype == BF and name in TUNED)
    slot, pos = [0, 0, 1, 0, 1, 0, 0, 1, 0], [0, 1, 129, 63, 64, 65, 199, 127, 128]
    q, qp = case.queries(len(pos))
    g, gp = _gate(case, len(pos))
    for ns in (1, 3, 7):
        got = _absorbed(case, slot, pos, qp, ns, gate=gp)
        close(case.unpad(got), case.want(q, slot, pos, g), 1.5e-2 if dtype == BF else 3e-6, f"{name} ns={ns}")
    idx = torch.tensor([8, 2, 5], dtype=torch.int32, device=DEV)
    got = _absorbed(case, slot, pos, qp, 2, index=idx)
    pick = idx.cpu().long()
    close(case.unpad(got)[pick], case.want(q, slot, pos)[pick], 1.5e-2 if dtype == BF else 3e-6, "indexed rows")
    rest = torch.ones(len(pos), dtype=torch.bool)
    rest[pick] = False
    assert not got.cpu()[rest].any()


@pytest.mark.parametrize("name", [n for n in TUNED if n != "r512_many"] + ["plain_wide"])
def test_one_key_stands_out(name):
    """A key aligned with every head's query outweighs all others: wherever it lies, rows that see it
    return its value, and the row just before it must not."""
    s = SIZES[name]
    for far in (0, 1, 62, 63, 64, 65, 126, 127, 128, 190):
        case = Case(s, [200], BF, sharp=0.02)
        q, qp = case.queries(3)
        case.kr[0][far] = 0
        loud = torch.zeros(s.rot_dim)
        loud[0] = 40.0 / s.scale ** 0.5  # entry 0 of the shared rotated part, already turned
        case.kr[0][far] = loud.to(BF)
        pg, r = int(case.table[0, far // 64]), far % 64
        case.cache[pg, r, s.krp:s.krp + s.rot_dim] = case.kr[0][far].to(DEV)
        pos = [max(far - 1, 0), far, 199]
        for i, p in enumerate(pos):  # queries whose turned entry 0 points at it
            v = torch.zeros(1, s.heads, s.rot_dim, dtype=torch.float64)
            v[..., 0] = 1.0 / s.scale ** 0.5
            q[i, :, s.dim:] = P.rotate(v, torch.tensor([-p]), s.rot_base, s.rot_dims)[0].to(BF)
        qp.view(3, -1)[:, :s.heads * (s.dkp + s.rp)].view(3, s.heads, -1)[..., s.dkp:s.dkp + s.rot_dim] = q[..., s.dim:].to(DEV)
        got = case.unpad(_absorbed(case, [0] * 3, pos, qp, 3))
        want = case.want(q, [0] * 3, pos)
        alone = torch.einsum("k,hvk->hv", case.c[0][far].double(), case.t["uv"].double().view(s.heads, s.vdim, -1)).reshape(-1)
        close(want[1], alone, 1e-6, "the oracle sees the loud key")
        close(got, want, 1.5e-2, f"{name} far={far}")
        if far:
            assert (got[0].double().cpu() - alone).norm() > 0.3 * alone.norm()


@pytest.mark.parametrize("name", ["small", "two_tiles", "r128", "r256", "r512", "r512_many"])
def test_expanded_attention(name):
    """Portions that start at 0 and inside a page, cut into tiles of several heights; gate applied."""
    from llm_sharding_amd.ops import latent as L
    from llm_sharding_amd.runtime.latent_mixer import Group
    s = SIZES[name]
    case = Case(s, [200, 130], BF)
    assert case.w.expand
    runs = [(0, 90, 0, 110), (90, 130, 1, 0), (220, 2, 0, 63)]
    slot = [r[2] for r in runs for _ in range(r[1])]
    pos = [r[3] + i for r in runs for i in range(r[1])]
    rows = len(pos)
    q, qp = case.queries(rows)
    g, gp = _gate(case, rows)
    want = case.want(q, slot, pos, g)
    a = case.args(slot, pos)
    for tile in (16, 64, 128):
        grp = Group(runs, tile, DEV)
        lat = torch.zeros(grp.tokens, s.cache_width, dtype=BF, device=DEV)
        kv = torch.zeros(grp.tokens, case.w.kv.n, dtype=BF, device=DEV)
        out = torch.zeros(rows, case.w.out.k, dtype=BF, device=DEV)
        L.gather(a, grp.src, grp.tokens, lat)
        assert torch.equal(lat[:200, :s.kv_rank].cpu(), case.c[0]) and torch.equal(lat[200:330, :s.kv_rank].cpu(), case.c[1])
        case.w.kv(lat, grp.tokens, kv)
        L.prefill(a, grp.tiles, grp.tiles_host, qp, kv, lat, gp, out, rows, grp.tokens)
        close(case.unpad(out), want, 1.5e-2, f"{name} tile={tile}")
    with pytest.raises(ValueError):
        L.prefill(a, grp.tiles, grp.tiles_host, qp, kv, lat, gp, out, rows, grp.tokens - 1)


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("name", ["small", "two_tiles", "r128", "r512", "wave_wide"])
def test_append_norms_turns_and_places(dtype, name):
    from llm_sharding_amd.ops import latent as L
    s = LatentSpec(2, 32, 16, 32, 504, 3080, 1e4, 16, 0.2) if name == "wave_wide" else SIZES[name]
    case = Case(s, [130, 70], dtype)
    slot, pos = [0, 1, 0, 0, 1], [129, 64, 63, 0, 127]
    w = case.w
    from llm_sharding_amd.runtime.blocks import InputProjection
    proj = InputProjection(w.input_parts(), "inp", 128)
    ok = proj.col["dkv"]
    inp = _rand(6, proj.lin.n, seed=3, dtype=dtype).to(DEV)
    cq = torch.zeros(6, w.uq.k, dtype=dtype, device=DEV)
    before = case.cache.clone()
    slot, pos = slot + [1], pos + [case.max_pages * 64]  # outside the table: nothing is written
    a = case.args(slot, pos)
    L.append(a, 6, inp, proj.col["dq"], ok, w.gq, w.gk, cq)
    x = inp.double().cpu()
    tol = 5e-3 if dtype == BF else 2e-6
    close(cq[:, :s.q_rank], P.gain_norm(x[:, :s.q_rank], case.t["dq.norm"].double(), 1e-4), tol, "query latent")
    d = x[:, ok:ok + s.kv_rank + s.rot_dim]
    c = P.gain_norm(d[:, :s.kv_rank], case.t["dkv.norm"].double(), 1e-4)
    kr = P.rotate(d[:, s.kv_rank:], torch.tensor(pos), s.rot_base, s.rot_dims)
    touched = torch.zeros(case.cache.shape[:2], dtype=torch.bool)
    for i in range(4):  # (row 4's page does not exist: slot 1 ends at page 1, so it does)
        pg = int(case.table[slot[i], pos[i] // 64])
        e = case.cache[pg, pos[i] % 64]
        close(e[:s.kv_rank], c[i], tol, f"latent of row {i}")
        close(e[s.krp:s.krp + s.rot_dim], kr[i], tol, f"rotated part of row {i}")
        assert not e[s.kv_rank:s.krp].any() and not e[s.krp + s.rot_dim:].any()
        touched[pg, pos[i] % 64] = True
    pg = int(case.table[1, 1])
    touched[pg, 63] = True
    assert torch.equal(case.cache.cpu()[~touched], before.cpu()[~touched])


# ------------------------------------------------------------------------------ engine
@pytest.fixture(scope="module")
def ordinary():
    cfg = M.stack()
    return cfg, M.tensors(cfg)


@pytest.fixture(scope="module")
def sharp():
    cfg = M.stack(sharp=3.0)
    return cfg, M.tensors(cfg)


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("sizes", [[300], [64, 1, 63, 66, 128], [2, 3, 2], [100, 65, 1, 1, 1], [1]])
def test_portions(ordinary, dtype, sizes):
    cfg, t = ordinary
    ids = _ids(300 if sizes[0] > 3 else 140)
    want = P.run(cfg.to_dict(), t, ids)
    eng = M.engine(cfg, DEV, dtype)
    got = torch.cat([M.feed(eng, [(1, p)]) for p in M.cut(ids, sizes)])
    assert M.rel(got, want) < TOL[dtype]


def test_portions_whose_softmax_picks_single_keys(sharp):
    cfg, t = sharp
    ids = _ids(330, seed=2)
    want = P.run(cfg.to_dict(), t, ids)
    for sizes in ([330], [190, 1, 2, 63], [37, 37, 3]):
        eng = M.engine(cfg, DEV, F32)
        got = torch.cat([M.feed(eng, [(0, p)]) for p in M.cut(ids, sizes)])
        assert M.rel(got, want) < SHARP_TOL, sizes


@pytest.mark.parametrize("dtype", [BF, F32])
def test_long_decoding(ordinary, dtype):
    """A two-token prompt, then 330 single tokens across five pages."""
    cfg, t = ordinary
    ids = _ids(332, seed=5)
    want = P.run(cfg.to_dict(), t, ids)
    eng = M.engine(cfg, DEV, dtype)
    got = [M.feed(eng, [(3, ids[:2])])] + [M.feed(eng, [(3, [x])]) for x in ids[2:]]
    assert M.rel(torch.cat(got), want) < TOL[dtype]


@pytest.mark.parametrize("dtype", [BF, F32])
def test_unequal_batches_on_reused_pages(ordinary, dtype):
    """Portions (expanded and short) beside decoded tokens, a pool that only holds the live requests, and
    a request on pages that two others filled before."""
    cfg, t = ordinary
    eng = M.engine(cfg, DEV, dtype, cache_tokens=64 * 10)
    seqs = {k: _ids(n, seed=k) for k, n in ((0, 260), (1, 75), (2, 200), (3, 140), (4, 3))}
    want = {k: P.run(cfg.to_dict(), t, v) for k, v in seqs.items()}
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
    with pytest.raises(RuntimeError):
        M.feed(eng, [(slot[3], seqs[3] * 2)])
    eng.reset([slot[3]])
    step([(0, 57), (2, 66), (4, 1)])
    eng.reset([slot[0], slot[2]])
    step([(3, 65), (4, 2)])
    step([(3, 75)])
    for k in seqs:
        assert at[k] == len(seqs[k]) and M.rel(torch.cat(got[k]), want[k]) < TOL[dtype], k


def test_rows_do_not_depend_on_the_batch(ordinary):
    """The same decoded token alone and among others, on other pages and in another slot."""
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
    assert M.rel(b[-1:], a) < TOL[F32]


def test_other_sizes_and_values_that_often_coincide():
    """Sizes beyond the tuned kernels, one layer without shared parts, scale 1, limit 1, base 1."""
    cfg = D.make_config(130, 129, [D.layer_entry(2, 130, 66, 200, 520, 131, ff=129, limit=1.0, base=1.0, rot_dims=2),
                                   D.layer_entry(7, 64, 64, 64, 64, 64, ff=64, scale=1.0),
                                   D.layer_entry(1, 1, 2, 1, 1, 1, ff=1, limit=0.1)], eps=0.5, embed_scale=1.0)
    t = M.tensors(cfg)
    ids = _ids(150, vocab=129)
    want = P.run(cfg.to_dict(), t, ids)
    for dtype, tol in ((F32, SHARP_TOL), (BF, 0.15)):
        eng = M.engine(cfg, DEV, dtype)
        got = torch.cat([M.feed(eng, [(0, p)]) for p in M.cut(ids, [100, 1, 49])])
        assert M.rel(got, want) < tol, dtype


def test_layers_of_a_real_width():
    """Wide heads and latents: portions on every projection kernel (1..16, 17..128, more rows), absorbed
    and expanded attention, groups of heads."""
    cfg = D.make_config(512, 260, [D.layer_entry(40, 128, 64, 128, 512, 256, ff=600),
                                   D.layer_entry(16, 128, 64, 128, 256, 128)])
    t = M.tensors(cfg)
    ids = _ids(350, vocab=260)
    want = P.run(cfg.to_dict(), t, ids, dtype=torch.float32)
    eng = M.engine(cfg, DEV, BF)
    got = torch.cat([M.feed(eng, [(0, p)]) for p in M.cut(ids, [100, 1, 20, 64, 129, 2, 34])])
    assert M.rel(got, want) < TOL[BF]


# ------------------------------------------------------------------------------ generation
@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("graph", [True, False])
def test_greedy_generation_through_the_server(sharp, ordinary, dtype, graph):
    """More requests than slots over a small page pool, prompts cut at the prefill budget, decode graphs
    replayed while slots come and go: fp32 engines give the plain evaluation's tokens, bf16 ones too
    where its choice is clear."""
    cfg, t = ordinary
    prompts = [_ids(n, seed=20 + n) for n in (4, 130, 1, 65, 33, 90, 7)]
    srv = PipelineServer(cfg, M.NamedSource(cfg, 0), device=DEV, batch=2, microbatches=2, max_seq=192, prefill_budget=100,
                         dtype=dtype, use_graph=graph, cache_tokens=64 * 7)
    outs = srv.generate(prompts, 8, eos_ids=())
    for p, o in zip(prompts, outs):
        want, gaps = P.greedy(cfg.to_dict(), t, p, 8)
        clear = next((i for i, gp in enumerate(gaps) if gp < (0.4 if dtype == BF else 1e-3)), 8)
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


def test_graph_replays_equal_eager_steps(ordinary):
    from llm_sharding_amd.runtime.engine import DecodeGraph
    cfg, _ = ordinary
    prompts = [_ids(60, seed=1), _ids(62, seed=2), _ids(3, seed=3)]
    a, b = M.engine(cfg, DEV, BF), M.engine(cfg, DEV, BF)
    for eng in (a, b):
        M.feed(eng, [(i, p) for i, p in enumerate(prompts)])
    g = DecodeGraph(a, 3, "full", history_len=8)
    tok = torch.tensor([5, 6, 7], dtype=torch.int32)
    g.tokens.copy_(tok)
    g.capture()
    for i in range(8):  # crosses a page border
        g.replay()
        M.feed(b, [(3, [i + 1])])  # the eager engine's own work in between
        torch.cuda.synchronize()
        slot, pos = b.prefill_rows([0, 1, 2], [1, 1, 1])
        h = b.forward(b.embed(tok), slot, pos)
        b.advance([0, 1, 2], [1, 1, 1])
        lg, tok = b.logits(h).cpu(), b.head(h).to(torch.int32).cpu()
        got = g.history[i].cpu()
        best = lg.max(-1).values - lg.gather(1, got.long()[:, None])[:, 0]
        assert float(best.max()) <= 2e-2 * float(lg.abs().max()), i
        g.tokens.copy_(tok)


def test_stages_on_one_gpu(ordinary):
    """Two and three pipeline stages (split head, captured graphs, fp32 stream between them) give the
    single engine's tokens."""
    from llm_sharding_amd.parallel.pipeline import drive_local_pipeline, run_pipeline_generate
    from llm_sharding_amd.config import get_preset
    cfg = get_preset("tiny-deretar")
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
    cfg, _ = ordinary
    folder = D.write_random_checkpoint(cfg, str(tmp_path / "m"), seed=0)
    want = P.run(cfg.to_dict(), M.tensors(cfg), _ids(70))
    ids = _ids(70)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": ids[:66], "want": [0, 65]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": ids[:2], "want": []}, {"id": "a", "tokens": ids[66:67], "want": []}],
              "end": ["b"]},
             {"step": 2, "entries": [{"id": "c", "tokens": ids[:1], "want": [0]}, {"id": "a", "tokens": ids[67:], "want": [2]}],
              "end": ["a", "c"]}]
    import json
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", "float32",
                        "--out", str(tmp_path), "--max-tokens", "200"], input="\n".join(map(json.dumps, steps)),
                       capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 2"]

    def read(n):
        return torch.frombuffer(bytearray((tmp_path / f"{n}.f32").read_bytes()), dtype=torch.float32).view(-1, cfg.vocab_size)

    assert not (tmp_path / "1.f32").exists()
    assert M.rel(read(0), want[[0, 65]]) < TOL[F32] and M.rel(read(2), want[[0, 69]]) < TOL[F32]
