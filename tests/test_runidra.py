"""Runidra on the CPU: configuration, checkpoint loading, placement, the stack engine's step function against
the plain evaluation (tests/plain_runidra.py), serving and pipelining, and that the plain evaluation itself
notices mistakes."""
import dataclasses
import json

import pytest
import torch

import plain_runidra as P
import runidra_models as M
from llm_sharding_amd.config import get_preset
from llm_sharding_amd.models import runidra as D
from llm_sharding_amd.models.stack import GluSpec, LatentSpec, MlstmSpec, MoeSpec
from llm_sharding_amd.parallel.pipeline import run_pipeline_generate
from llm_sharding_amd.parallel.server import PipelineServer
from llm_sharding_amd.runtime import registry as R

TOL = 5e-5


def _ids(n, vocab=150, seed=0):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


@pytest.fixture(scope="module")
def model():
    cfg = M.stack(sharp=3.0)
    return cfg, M.tensors(cfg)


# ------------------------------------------------------------------------------ configuration
def test_config_is_read_layer_by_layer():
    cfg = M.stack()
    assert [s.owner for s in cfg.layers] == [0, 1, 2, 1, 2, 3, 4, 5] and not any(s.enters is not None for s in cfg.layers)
    assert cfg.layers[1] == cfg.layers[3] and cfg.layers[5].mlp is None and cfg.layers[7].mlp is None
    assert cfg.layers[0].mixer == MlstmSpec(3, 20, 28, 6.0, 20 ** -0.5) and cfg.layers[0].mixer.state_dims == (32, 32)
    assert cfg.layers[1].mixer == LatentSpec(5, 24, 16, 40, 48, 72, 500.0, 16, 40 ** -0.5, gate=False, window=37, sink=True,
                                             interleaved=True)
    assert cfg.layers[0].mlp == GluSpec(90, gelu=True, bias=True)
    assert cfg.layers[1].mlp == MoeSpec(6, 2, 40, shared_ff=50, shared_gate=True, bias=True)
    assert (cfg.streams, cfg.stream_width, cfg.stream_bytes()) == (3, 264, 1056)
    assert (cfg.logit_scale, cfg.logit_softcap, cfg.norm_eps, cfg.tie_word_embeddings) == (0.7, 9.0, 0.02, False)
    again = D.config_from_dict(json.loads(json.dumps(cfg.to_dict())))
    assert again.layers == cfg.layers and again.streams == 3
    assert [s.owner for s in D.config_from_dict({**cfg.to_dict(), "loop": None}).layers] == list(range(6))
    assert D.config_from_dict({**cfg.to_dict(), "loop": {"start": 0, "stop": 6, "times": 1}}).num_hidden_layers == 6
    assert D.config_from_dict({**cfg.to_dict(), "loop": {"start": 5, "stop": 6, "times": 4}}).num_hidden_layers == 9


def test_config_refuses_what_the_design_does_not_have():
    def changed(i, **kw):
        d = json.loads(json.dumps(M.stack().to_dict()))
        for k, v in kw.items():
            d["layers"][i][k] = {**d["layers"][i][k], **v} if isinstance(v, dict) and d["layers"][i][k] else v
        return d

    base = M.stack().to_dict()
    for bad in (changed(0, type="other"), changed(0, mlp={"kind": "sparse"}), changed(0, mixer={"gate_cap": 0}),
                changed(0, mixer={"heads": 0}), changed(1, mixer={"mask": {"size": 0}}), changed(1, mlp={"router": {"experts": 2, "top": 3}}),
                changed(1, mixer={"rot": {"base": 10.0, "dims": 18}}), changed(1, mixer={"rot": {"base": 10.0, "dims": 7}}),
                changed(0, mlp={"ff": 0}), {**base, "streams": 0}, {**base, "logit_softcap": -1.0},
                {**base, "loop": {"start": 3, "stop": 3, "times": 2}}, {**base, "loop": {"start": 0, "stop": 7, "times": 1}},
                {**base, "layers": []}):
        with pytest.raises(ValueError):
            D.config_from_dict(bad)


def test_registry_reads_a_checkpoint(tmp_path):
    cfg = M.stack()
    folder = D.write_random_checkpoint(cfg, str(tmp_path / "m"), seed=4)
    got = R.load_config(folder)
    assert R.is_stack(got) and got.layers == cfg.layers and R.engine_class(got).__name__ == "StackEngine"
    assert R.kernel_family(got) == "streams"
    src, want = R.folder_source(folder, got), M.tensors(cfg, seed=4)
    a, b = (src.layer(i, "cpu", torch.bfloat16) for i in (2, 4))  # two runs of layer 2
    assert torch.equal(a["hc2.mix"], want["l2.hc2.mix"]) and torch.equal(a["mix.v"], b["mix.v"])
    assert torch.equal(src.lm_head("cpu", torch.bfloat16), want["head"])
    one = got.layers[0]
    got.layers[0] = dataclasses.replace(one, mixer=dataclasses.replace(one.mixer, vdim=41))
    with pytest.raises(ValueError):
        src.layer(0, "cpu", torch.bfloat16)


def test_placement_counts_streams_and_states():
    from llm_sharding_amd.parallel.scheduler import plan_stages, stage_memory
    cfg = M.stack()
    assert cfg.stage_cuts() == list(range(8)) and len(plan_stages(cfg, 4).ranges()) == 4
    big = get_preset("runidra-4k")
    s = big.layers[0].mixer
    assert (s.state_dims, s.copies, s.state_bytes) == ((128, 128), 2, 4 * 32 * (128 * 128 + 2 * 129))
    assert big.num_hidden_layers == 34 and big.kv_bytes_per_token_per_layer() == 2 * 576
    assert big.state_bytes_per_slot() == s.state_bytes and big.stream_bytes() == 4 * 4 * 4096
    m = stage_memory(big, 8, slots=4, max_seq=1024, prefill_rows=2048)
    assert m["kv"] == 8 * 4 * (1024 * 576 * 2 + s.state_bytes)
    t = M.tensors(cfg)
    for i, l in enumerate(cfg.layers):
        assert cfg.layer_params(i) == sum(v.numel() for k, v in t.items() if k.startswith(f"l{l.owner}.")), i


def test_gated_units_refuse_what_no_kernel_has():
    for kw in (dict(gelu=True, limit=1.0), dict(bias=True), dict(limit=-1.0)):
        with pytest.raises(ValueError):
            GluSpec(8, **kw)


# ------------------------------------------------------------------------------ engine (CPU)
def test_whole_portions_and_decoding_agree(model):
    cfg, t = model
    ids = _ids(150)
    want = P.run(cfg.to_dict(), t, ids)
    for sizes in ([150], [64, 1, 63, 22], [2, 3], [1]):
        eng = M.engine(cfg, "cpu", torch.float32)
        got = torch.cat([M.feed(eng, [(2, part)]) for part in M.cut(ids, sizes)])
        assert M.rel(got, want) < TOL, sizes


def test_batches_reused_pages_and_slots(model):
    cfg, t = model
    eng = M.engine(cfg, "cpu", torch.float32, cache_tokens=64 * 5)
    a, b, c = _ids(100, seed=1), _ids(130, seed=2), _ids(70, seed=3)
    wa, wb, wc = (P.run(cfg.to_dict(), t, x) for x in (a, b, c))
    ga, gb = [], []
    for pa, pb in ((a[:60], b[:1]), (a[60:61], b[1:120]), (a[61:], b[120:])):
        lg = M.feed(eng, [(1, pa), (0, pb)])
        ga.append(lg[:len(pa)])
        gb.append(lg[len(pa):])
    assert M.rel(torch.cat(ga), wa) < TOL and M.rel(torch.cat(gb), wb) < TOL
    with pytest.raises(RuntimeError):
        M.feed(eng, [(3, c)])  # the pool is taken
    eng.reset([1])
    assert M.rel(M.feed(eng, [(1, c)]), wc) < TOL  # the slot's old state does not show
    eng.reset()
    assert len(eng.pool.free) == eng.pool.pages


def test_stages_hand_each_other_all_streams(model):
    cfg, t = model
    ids = _ids(40)
    stages = [M.engine(cfg, "cpu", torch.float32, start=a, end=b) for a, b in ((0, 2), (2, 7), (7, 8))]
    slot, pos = stages[0].prefill_rows([0], [40])
    h = stages[0].embed(torch.tensor(ids))
    assert h.shape == (40, cfg.stream_width)
    for e in stages:
        h = e.forward(h, slot, pos)
    assert M.rel(stages[-1].logits(h), P.run(cfg.to_dict(), t, ids)) < TOL


def test_a_key_just_inside_and_just_outside_the_window():
    for window in (1, 7, 64, 65):
        cfg, t = M.asking(window)
        eng = M.engine(cfg, "cpu", torch.float32, t=t)
        for far in (0, 3, 63, 64):
            ids = _ids(far + window + 3, vocab=148, seed=far)
            ids[far] = M.LOUD
            ids[far + window - 1] = M.ASK if window > 1 else M.LOUD
            ids[far + window] = ids[far + window + 1] = M.ASK
            eng.reset([0])
            got = torch.cat([M.feed(eng, [(0, p)]) for p in (ids[:far + window - 1], *([x] for x in ids[far + window - 1:])) if p])
            want = P.run(cfg.to_dict(), t, ids)
            assert M.rel(got, want) < TOL
            narrow = {**cfg.to_dict()["layers"][0]["mixer"], "mask": {"size": window + 1}}
            d = {**cfg.to_dict(), "layers": [{**cfg.to_dict()["layers"][0], "mixer": narrow}]}
            off = P.run(d, t, ids)[far + window] - want[far + window]
            assert float(off.norm() / want[far + window].norm()) > 0.1  # one token more would show


def test_server_schedules_over_a_small_pool(model):
    """More requests than slots and pages: admission waits for pages, prompts are cut at the budget, slots and
    their states are used again."""
    cfg, t = model
    prompts = [_ids(n, seed=10 + n) for n in (5, 70, 1, 33, 90, 20)]
    srv = PipelineServer(cfg, M.NamedSource(cfg, 0), device="cpu", batch=2, microbatches=2, max_seq=128,
                         prefill_budget=24, dtype=torch.float32, cache_tokens=64 * 3)
    outs = srv.generate(prompts, 5, eos_ids=())
    for p, o in zip(prompts, outs):
        want, gaps = P.greedy(cfg.to_dict(), t, p, 5)
        assert o == want, (len(p), gaps)
    assert len(srv.eng.pool.free) == 3


def test_pipeline_generates(model):
    cfg, t = model
    prompts = torch.tensor([_ids(6, seed=s) for s in range(4)]).view(2, 2, 6)
    out = run_pipeline_generate(cfg, M.NamedSource(cfg, 0), prompts, 4, 0, 1, batch=2, microbatches=2, max_seq=64,
                                dtype=torch.float32)
    for i in range(4):
        want, gaps = P.greedy(cfg.to_dict(), t, prompts.view(4, 6)[i].tolist(), 4)
        assert out.permute(1, 2, 0).reshape(4, -1)[i].tolist() == want, gaps


def test_command_line_generates(monkeypatch):
    """inference.py takes this design like any other."""
    import os
    import sys
    monkeypatch.syspath_prepend(os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
    import inference
    cfg = get_preset("tiny-runidra")
    tok = inference.SyntheticByteTokenizer(cfg.vocab_size)
    ids = tok("a few words", return_tensors="pt")["input_ids"][0].tolist()
    monkeypatch.setattr(sys, "argv", ["inference.py", "--random", "tiny-runidra", "--prompt", "a few words",
                                      "--max-new-tokens", "5", "--device", "cpu"])
    want, gaps = P.greedy(cfg.to_dict(), D.random_tensors(cfg, 0, torch.float32), ids, 5)
    assert inference.main() == want, gaps


# ------------------------------------------------------------------------------ the oracle notices
def _mistakes():
    window, rotate, memory, route, scatter, order, unit = P.window, P.rotate, P.memory, P.route, P.scatter, P.order, P.unit

    def halves(x, rot):  # pairs (i, i + dims / 2)
        n = rot["dims"]
        at = [j for i in range(n // 2) for j in (i, i + n // 2)]
        out = x.clone()
        out[..., at] = rotate(x[..., at + list(range(n, x.shape[-1]))], rot)[..., :n]
        return out

    def stale(q, k, v, i, f, state=None):  # the read-out before the write
        S, z, m = (torch.zeros(k.shape[1], v.shape[1], dtype=k.dtype), torch.zeros(k.shape[1], dtype=k.dtype), torch.zeros((), dtype=k.dtype))
        out = torch.empty_like(v)
        for t in range(k.shape[0]):
            out[t] = (S.T @ q[t]) / P.denominator(z @ q[t], m)
            _, (S, z, m) = memory(q[t:t + 1], k[t:t + 1], v[t:t + 1], i[t:t + 1], f[t:t + 1], (S, z, m))
        return out

    return {
        "window_narrow": ("window", lambda n, s: window(n, s - 1)),
        "window_wide": ("window", lambda n, s: window(n, s + 1)),
        "no_sink": ("sink_softmax", lambda s, sink: torch.softmax(s, -1)),
        "sink_of_zero": ("sink_softmax", lambda s, sink: torch.softmax(torch.cat([s, torch.zeros_like(s[:, :1])], -1), -1)[:, :-1]),
        "rotate_none": ("rotate", lambda x, rot: x),
        "rotate_halves": ("rotate", halves),
        "capped": ("capped", lambda z, cap: z),
        "memory_stale": ("memory", lambda *a: (stale(*a), None)),
        "denominator_without_floor": ("denominator", lambda nq, m: nq.abs() + 1e-6),
        "denominator_signed": ("denominator", lambda nq, m: torch.maximum(nq, torch.exp(-m)) + 1e-6),
        "denominator_none": ("denominator", lambda nq, m: torch.exp(-m)),
        "memory_no_forgetting": ("memory", lambda q, k, v, i, f, state=None: memory(q, k, v, i, 0 * f)),
        "memory_even_gates": ("memory", lambda q, k, v, i, f, state=None: memory(q, k, v, 0 * i, f)),
        "scatter_transposed": ("scatter", lambda xs, mix, out, y: scatter(xs, mix.T, out, y)),
        "scatter_even": ("scatter", lambda xs, mix, out, y: scatter(xs, mix, torch.ones_like(out), y)),
        "gather_even": ("gather", lambda xs, w: xs.sum(1)),
        "leave_first": ("leave", lambda xs: xs[:, 0]),
        "route_even": ("route", lambda z, top: (route(z, top)[0], torch.full_like(route(z, top)[1], 1 / top))),
        "gelu": ("gelu", P.silu),
        "silu": ("silu", P.gelu),
        "unit_without_bias": ("unit", lambda h, w, act: unit(h, {k: x for k, x in w.items() if not k.endswith(".b")}, act)),
        "order_once": ("order", lambda cfg: order({**cfg, "loop": None})),
    }


@pytest.mark.parametrize("name", list(_mistakes()))
def test_a_planted_mistake_shows(model, name, monkeypatch):
    cfg, t = model
    ids = _ids(110)
    good = P.run(cfg.to_dict(), t, ids)
    fn, bad = _mistakes()[name]
    monkeypatch.setattr(P, fn, bad)
    assert M.rel(P.run(cfg.to_dict(), t, ids), good) > 20 * TOL, name


def test_chunk_form_equals_steps():
    """The equations of the chunked kernel, in float64: chunks and segments against token by token."""
    g = torch.Generator().manual_seed(3)
    n, dk, dv = 50, 12, 10
    q, k = (torch.randn(n, dk, generator=g, dtype=torch.float64) for _ in range(2))
    v = torch.randn(n, dv, generator=g, dtype=torch.float64)
    i, f = torch.randn(n, generator=g, dtype=torch.float64) * 4, -torch.rand(n, generator=g, dtype=torch.float64) * 3
    state = (torch.randn(dk, dv, generator=g, dtype=torch.float64), torch.randn(dk, generator=g, dtype=torch.float64),
             torch.tensor(1.5, dtype=torch.float64))
    want, (S1, z1, m1) = P.memory(q, k, v, i, f, state)

    def chunk(q, k, v, i, f, S, z, m):
        F = f.cumsum(0)
        gs = i - F
        Mx = torch.maximum(m, gs.cummax(0).values)
        w = torch.tril(torch.exp(gs[None] - Mx[:, None])) * (q @ k.T)
        keep = torch.exp(m - Mx)
        nq = keep * (q @ z) + w.sum(1)
        out = (keep[:, None] * (q @ S) + w @ v) / (torch.maximum(nq.abs(), torch.exp(-(F + Mx))) + 1e-6)[:, None]
        a, b = torch.exp(m - Mx[-1]), torch.exp(gs - Mx[-1])
        return out, a * S + (k * b[:, None]).T @ v, a * z + (k * b[:, None]).sum(0), F[-1] + Mx[-1], F[-1]
    out, S, z, m, _ = chunk(q, k, v, i, f, *state)
    assert torch.allclose(out, want) and torch.allclose(S, S1) and torch.allclose(z, z1) and torch.allclose(m, m1)
    # a segment from an empty state, then joined to what lies before it
    none = (torch.zeros(dk, dv, dtype=torch.float64), torch.zeros(dk, dtype=torch.float64), torch.tensor(-torch.inf, dtype=torch.float64))
    _, Sa, za, ma, fa = chunk(*(x[:20] for x in (q, k, v, i, f)), *none)
    top = torch.maximum(state[2] + fa, ma)
    keep, add = torch.exp(state[2] + fa - top), torch.exp(ma - top)
    out, S, z, m, _ = chunk(*(x[20:] for x in (q, k, v, i, f)), keep * state[0] + add * Sa, keep * state[1] + add * za, top)
    assert torch.allclose(out, want[20:]) and torch.allclose(S, S1) and torch.allclose(z, z1) and torch.allclose(m, m1)
