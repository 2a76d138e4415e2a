"""Gupuvik on the CPU: configuration, checkpoint loading, placement, the stack engine's step function against
the plain evaluation (tests/plain_gupuvik.py), serving and pipelining, and that the plain evaluation itself
notices mistakes."""
import dataclasses
import json

import pytest
import torch

import gupuvik_models as M
import plain_gupuvik as P
from llm_sharding_amd.config import get_preset
from llm_sharding_amd.models import gupuvik as G
from llm_sharding_amd.models.stack import AttentionSpec, DeltaSpec, DenseSpec, MoeSpec
from llm_sharding_amd.ops.delta import CHUNK, chunk_groups
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
    kinds = [type(s.mixer) for s in cfg.layers]
    assert kinds == [DeltaSpec, AttentionSpec, AttentionSpec, DeltaSpec, AttentionSpec, AttentionSpec, DeltaSpec]
    assert [getattr(s.mixer, "kv_from", None) for s in cfg.layers] == [None, None, 1, None, None, 1, None]
    assert [type(s.mlp) for s in cfg.layers] == [MoeSpec, DenseSpec, MoeSpec, type(None), type(None), MoeSpec, DenseSpec]
    a, d = cfg.layers[2].mixer, cfg.layers[3].mixer
    assert (a.window, a.keep_first, a.softcap) == (70, 0, 9.0) and (d.taps, d.dim, d.vdim) == (5, 36, 70)
    assert d.q_scale == 36 ** -0.5 and d.state_dims == (64, 128) and cfg.layers[6].mixer.state_dims == (33, 129)
    again = G.config_from_dict(json.loads(json.dumps(cfg.to_dict())), rank=M.RANK)
    assert again.layers == cfg.layers and (again.embed_scale, again.norm_eps) == (1.7, 1e-5)
    assert not again.tie_word_embeddings


def test_config_refuses_what_the_design_does_not_have():
    def changed(i, **kw):
        d = json.loads(json.dumps(M.stack().to_dict()))
        for k, v in kw.items():
            d["layers"][i][k] = {**d["layers"][i][k], **v} if isinstance(v, dict) and d["layers"][i][k] else v
        return d

    for bad in (changed(0, type="other"), changed(1, mlp={"kind": "sparse"}), changed(2, mixer={"kv_from": 0}),
                changed(2, mixer={"kv_from": 4}), changed(5, mixer={"kv_from": 2}), changed(2, mixer={"kv_from": 9}),
                changed(2, mixer={"vdim": 41}), changed(1, mixer={"kv_heads": 4}),
                changed(0, mlp={"router": {"experts": 5, "top": 6}})):
        with pytest.raises(ValueError):
            G.config_from_dict(bad)


def test_registry_reads_a_checkpoint(tmp_path):
    """The ranks come from the tensors: config.json does not have them."""
    cfg = M.stack()
    folder = G.write_random_checkpoint(cfg, str(tmp_path / "m"), seed=4)
    got = R.load_config(folder)
    assert R.is_stack(got) and got.layers == cfg.layers and R.engine_class(got).__name__ == "StackEngine"
    assert got.layers[0].mixer.decay_rank == got.layers[0].mixer.gate_rank == M.RANK
    src, want = R.folder_source(folder, got), M.tensors(cfg, seed=4)
    assert torch.equal(src.layer(3, "cpu", torch.bfloat16)["mix.a2"], want["l3.mix.a2"])
    assert "mix.k" not in src.layer(2, "cpu", torch.bfloat16)
    assert torch.equal(src.lm_head("cpu", torch.bfloat16), want["head"])
    assert torch.equal(src.embedding("cpu", torch.bfloat16), want["embed"])
    one = got.layers[3]
    got.layers[3] = dataclasses.replace(one, mixer=dataclasses.replace(one.mixer, vdim=71))
    with pytest.raises(ValueError):
        src.layer(3, "cpu", torch.bfloat16)


def test_placement_keeps_shared_keys_together():
    from llm_sharding_amd.parallel.scheduler import kv_slots_for_memory, plan_stages, stage_memory
    cfg = M.stack()
    assert cfg.stage_cuts() == [0, 1, 6]  # layers 2 and 5 read layer 1's keys
    assert plan_stages(cfg, 3).ranges() == [(0, 1), (1, 6), (6, 7)]
    with pytest.raises(ValueError):
        plan_stages(cfg, 4)
    big = get_preset("gupuvik-4k")
    for s in plan_stages(big, 4).stages:
        assert s.start in big.stage_cuts()
    st = big.state_bytes_per_slot()
    assert st == 4 * (32 * 128 * 128 + 4 * 3 * 32 * 128)
    assert stage_memory(big, 8, slots=32, max_seq=4096, prefill_rows=2048)["kv"] == 8 * 32 * (4096 * 2048 * 2 + st)
    assert kv_slots_for_memory(big, 8, 4096, 40e9, 20e9) == int((40e9 - 8e9 - 20e9) // (8 * (4096 * 2048 * 2 + st)))
    with pytest.raises(ValueError):
        M.engine(cfg, "cpu", torch.float32, start=2)


def test_long_runs_are_cut_into_groups_of_chunks():
    runs = [(0, 100, 2, 7), (100, 33, 0, 0), (133, 1000, 1, 64)]
    at = {r[2]: 0 for r in runs}
    for chunks, spans in chunk_groups(runs, 9):
        assert chunks.shape[0] <= 9
        for c0, n, slot, pos0, row0, rows, _, _ in spans.tolist():
            run = next(r for r in runs if r[2] == slot)
            assert (row0, pos0) == (run[0] + at[slot], run[3] + at[slot]) and n == -(-rows // CHUNK)
            for i, (r0, k, s, p0, before, *_) in enumerate(chunks[c0:c0 + n].tolist()):
                assert (r0, s, p0, before) == (row0 + i * CHUNK, slot, pos0 + i * CHUNK, at[slot] + i * CHUNK)
                assert k == min(CHUNK, rows - i * CHUNK)
            at[slot] += rows
    assert at == {2: 100, 0: 33, 1: 1000}


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


def test_stages_hand_each_other_the_stream(model):
    cfg, t = model
    ids = _ids(40)
    stages = [M.engine(cfg, "cpu", torch.float32, start=a, end=b) for a, b in ((0, 1), (1, 6), (6, 7))]
    slot, pos = stages[0].prefill_rows([0], [40])
    h = stages[0].embed(torch.tensor(ids))
    for e in stages:
        h = e.forward(h, slot, pos)
    assert M.rel(stages[-1].logits(h), P.run(cfg.to_dict(), t, ids)) < TOL


def test_server_schedules_over_a_small_pool(model):
    """More requests than slots and pages: admission waits for pages, prompts are cut at the budget, slots
    and their states are used again."""
    cfg, t = model
    prompts = [_ids(n, seed=10 + n) for n in (5, 70, 1, 33, 90, 20)]
    srv = PipelineServer(cfg, M.NamedSource(cfg, 0), device="cpu", batch=2, microbatches=2, max_seq=128,
                         prefill_budget=24, dtype=torch.float32, cache_tokens=64 * 3)
    outs = srv.generate(prompts, 5, eos_ids=())
    for p, o in zip(prompts, outs):
        want, gaps = P.greedy(cfg.to_dict(), t, p, 5)
        assert o == want, (len(p), gaps)
    assert len(srv.eng.pool.free) == 3
    with pytest.raises(ValueError):
        srv.request_replan([[0, 7], [7, 7]])


def test_replan_refuses_to_part_shared_keys(model):
    cfg, _ = model
    srv = PipelineServer(cfg, M.NamedSource(cfg, 0), rank=0, world=2, start=0, end=1, device="cpu", batch=1,
                         microbatches=1, max_seq=64, dtype=torch.float32)
    with pytest.raises(ValueError):
        srv.request_replan([[0, 3], [3, 7]])
    srv.request_replan([[0, 6], [6, 7]])


def test_pipeline_generates(model):
    cfg, t = model
    prompts = torch.tensor([_ids(6, seed=s) for s in range(4)]).view(2, 2, 6)
    out = run_pipeline_generate(cfg, M.NamedSource(cfg, 0), prompts, 4, 0, 1, batch=2, microbatches=2, max_seq=64,
                                dtype=torch.float32)
    for i in range(4):
        want, gaps = P.greedy(cfg.to_dict(), t, prompts.view(4, 6)[i].tolist(), 4)
        assert out.permute(1, 2, 0).reshape(4, -1)[i].tolist() == want, gaps


def test_reference_style_chain(tmp_path, model):
    """Two nodes of the TCP chain pass one request through by hand."""
    import socket

    from llm_sharding_amd.utils.node_worker import NodeWorker
    cfg, t = model
    folder = G.write_random_checkpoint(cfg, str(tmp_path / "m"), seed=0)
    ports = []
    for _ in range(2):
        with socket.socket() as sk:
            sk.bind(("127.0.0.1", 0))
            ports.append(sk.getsockname()[1])
    nodes = [NodeWorker(f"tcp://*:{ports[i]}", f"tcp://127.0.0.1:{ports[1 - i]}", i == 0, folder, dtype=torch.float32,
                        max_batch=1, max_seq=128, verbose=False) for i in range(2)]
    try:
        nodes[0].load_shards(0, 1)
        nodes[1].load_shards(1, 7)
        prompt = _ids(9, seed=6)
        want, _ = P.greedy(cfg.to_dict(), t, prompt, 4)
        state = nodes[0].receive_user_request(input_ids=torch.tensor([prompt]))
        got = []
        for _ in range(4):
            tok = nodes[1].pass_through_shard(nodes[0].pass_through_shard(state))
            got.append(int(tok))
            _, state = nodes[0].receive_next_token(tok)
        assert got == want
    finally:
        for n in nodes:
            n.close()


# ------------------------------------------------------------------------------ the oracle notices
def _mistakes():
    visible, delta_rule, short_conv, route, log_decay = P.visible, P.delta_rule, P.short_conv, P.route, P.log_decay

    def stale(q, k, v, decay, beta, state=None):  # the read-out before the write
        out, S = delta_rule(q, k, v, decay, beta, state)
        kq = (k * q).sum(-1, keepdim=True)
        return out - kq * beta[:, None] * v, S

    return {
        "visible_narrow": ("visible", lambda n, s, f: visible(n, s - 1, f)),
        "visible_wide": ("visible", lambda n, s, f: visible(n, s + 1, f)),
        "visible_first": ("visible", lambda n, s, f: visible(n, s, max(f - 1, 0))),
        "capped": ("capped", lambda s, cap: s),
        "head_gate": ("head_gate", lambda h, w: torch.ones(h.shape[0], w["g"].shape[0], dtype=h.dtype)),
        "unit": ("unit", lambda x: x),
        "delta_rule": ("delta_rule", stale),
        "short_conv": ("short_conv", lambda x, taps: short_conv(x, taps.flip(1))),
        "log_decay": ("log_decay", lambda h, w, m: log_decay(h, w, m).mean(-1, keepdim=True).expand(-1, -1, m["dim"])),
        "route": ("route", lambda z, top: (route(z, top)[0], torch.softmax(z, -1).gather(1, route(z, top)[0]))),
        "gelu": ("gelu", P.silu),
        "residual_gate": ("residual_gate", lambda h, w, b: torch.sigmoid(h @ w.T)),
        "scalar_norm": ("scalar_norm", lambda x, g, eps: P.rms(x, eps)),
    }


@pytest.mark.parametrize("name", list(_mistakes()))
def test_a_planted_mistake_shows(model, name, monkeypatch):
    cfg, t = model
    ids = _ids(90)
    good = P.run(cfg.to_dict(), t, ids)
    fn, bad = _mistakes()[name]
    monkeypatch.setattr(P, fn, bad)
    assert M.rel(P.run(cfg.to_dict(), t, ids), good) > 20 * TOL, name


def test_chunk_form_equals_steps():
    """The equations of the chunked kernels, in float64: one chunk against token by token."""
    g = torch.Generator().manual_seed(3)
    n, dk, dv = 32, 12, 10
    q, k = (P.unit(torch.randn(n, dk, generator=g, dtype=torch.float64)) for _ in range(2))
    v, S0 = torch.randn(n, dv, generator=g, dtype=torch.float64), torch.randn(dk, dv, generator=g, dtype=torch.float64)
    lg = -torch.rand(n, dk, generator=g, dtype=torch.float64) * 3
    beta = torch.rand(n, generator=g, dtype=torch.float64)
    want, S = P.delta_rule(q, k, v, lg.exp(), beta, S0)
    G_ = lg.cumsum(0)
    e = (G_[:, None] - G_[None]).exp()
    A = torch.tril(beta[:, None] * torch.einsum("id,ijd,jd->ij", k, e, k), -1)
    Pm = torch.tril(torch.einsum("id,ijd,jd->ij", q, e, k))
    T = torch.linalg.inv(torch.eye(n, dtype=torch.float64) + A)
    u = T @ (beta[:, None] * v) - T @ (beta[:, None] * k * G_.exp()) @ S0
    assert torch.allclose((q * G_.exp()) @ S0 + Pm @ u, want, atol=1e-10)
    assert torch.allclose(G_[-1].exp()[:, None] * S0 + (k * (G_[-1] - G_).exp()).T @ u, S, atol=1e-10)
