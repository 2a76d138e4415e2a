"""Deretar on the CPU: configuration, checkpoint loading, page pool, the stack engine's step function
against the plain evaluation (tests/plain_deretar.py), serving and pipelining, and that the plain
evaluation itself notices mistakes."""
import dataclasses
import json
import os
import subprocess
import sys

import pytest
import torch

import deretar_models as M
import plain_deretar as P
from llm_sharding_amd.config import get_preset
from llm_sharding_amd.models import deretar as D
from llm_sharding_amd.parallel.pipeline import run_pipeline_generate
from llm_sharding_amd.parallel.server import PipelineServer
from llm_sharding_amd.runtime import registry as R
from llm_sharding_amd.runtime.paging import PagePool

TOL = 2e-4  # ten times what fp32 rounding makes of these sharp softmaxes
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def _ids(n, vocab=150, seed=0):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


@pytest.fixture(scope="module")
def model():
    cfg = M.stack(sharp=3.0)
    return cfg, M.tensors(cfg)


# ------------------------------------------------------------------------------ configuration
def test_config_is_read_layer_by_layer():
    cfg = M.stack()
    assert [s.owner for s in cfg.layers] == [0, 1, 0, 3, 1, 5]
    assert cfg.layers[1].mlp is None and cfg.layers[3].mlp.limit == 0.75 and cfg.layers[3].mixer.rot_dims == 6
    again = D.config_from_dict(json.loads(json.dumps(cfg.to_dict())))
    assert again.layers == cfg.layers and again.embed_scale == 6.5 and again.norm_eps == 1e-5


def test_config_refuses_what_the_design_does_not_have():
    def changed(**kw):
        d = json.loads(json.dumps(M.stack().to_dict()))
        d["layers"][2].update(kw)
        return d

    for bad in (dict(type="window_attention"), dict(weights_of=2), dict(weights_of=9),
                dict(mlp={"kind": "dense", "ff": 91, "limit": 1.25}), dict(mlp={"kind": "sparse", "ff": 90, "limit": 1})):
        with pytest.raises(ValueError):
            D.config_from_dict(changed(**bad))
    with pytest.raises(ValueError):
        R.engine_class(M.stack())(M.stack(), 0, 1, "cpu", torch.float32, causal=False)


def test_registry_chooses_by_config(tmp_path):
    cfg = M.stack()
    folder = D.write_random_checkpoint(cfg, str(tmp_path / "m"), seed=4)
    got = R.load_config(folder)
    assert R.is_stack(got) and got.layers == cfg.layers and R.engine_class(got).__name__ == "StackEngine"
    src = R.folder_source(folder, got)
    want = M.tensors(cfg, seed=4)
    assert torch.equal(src.layer(4, "cpu", torch.bfloat16)["mix.uk"], want["l1.mix.uk"])  # the owner's tensors
    assert torch.equal(src.embedding("cpu", torch.bfloat16), want["embed"])
    lone = got.layers[3]
    got.layers[3] = dataclasses.replace(lone, mixer=dataclasses.replace(lone.mixer, kv_rank=199))
    with pytest.raises(ValueError):
        src.layer(3, "cpu", torch.bfloat16)  # a shape that config.json contradicts
    assert R.engine_class(get_preset("tiny")).__name__ == "StageEngine"
    with pytest.raises(ValueError):
        (tmp_path / "x").mkdir()
        (tmp_path / "x" / "config.json").write_text(json.dumps({"architecture": "Other", "layers": []}))
        R.load_config(str(tmp_path / "x"))


# ------------------------------------------------------------------------------ pages
def test_page_pool_gives_takes_and_gives_back():
    p = PagePool(pages=4, slots=3, max_seq=200, page_tokens=64)
    p.ensure(0, 65)
    p.ensure(1, 1)
    assert len(p.held[0]) == 2 and len(p.held[1]) == 1 and p.max_pages == 4
    assert p.table[0].tolist() == p.held[0] + [-1, -1]
    with pytest.raises(RuntimeError):
        p.ensure(2, 129)
    assert p.held[2] == []  # a refused request takes nothing
    old = list(p.held[0])
    p.release(0)
    p.ensure(2, 128)
    assert sorted(p.held[2]) == sorted(old) and p.table[0].tolist() == [-1] * 4
    with pytest.raises(ValueError):
        p.ensure(2, 257)


# ------------------------------------------------------------------------------ engine (CPU)
def test_whole_portions_and_decoding_agree(model):
    cfg, t = model
    ids = _ids(150)
    want = P.run(cfg.to_dict(), t, ids)
    for sizes in ([150], [64, 1, 63, 22], [2, 3], [1]):
        eng = M.engine(cfg, "cpu", torch.float32)
        got = torch.cat([M.feed(eng, [(2, part)]) for part in M.cut(ids, sizes)])
        assert M.rel(got, want) < TOL, sizes


def test_batches_and_reused_pages(model):
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
    assert M.rel(M.feed(eng, [(3, c)]), wc) < TOL


def test_stages_hand_each_other_the_stream(model):
    cfg, t = model
    ids = _ids(40)
    first = M.engine(cfg, "cpu", torch.float32, end=3)
    last = M.engine(cfg, "cpu", torch.float32, start=3)
    slot, pos = first.prefill_rows([0], [40])
    h = first.forward(first.embed(torch.tensor(ids)), slot, pos)
    assert h.dtype == first.hidden_dtype == torch.float32
    got = last.logits(last.forward(h, slot, pos))
    assert M.rel(got, P.run(cfg.to_dict(), t, ids)) < TOL


def test_server_schedules_over_a_small_pool(model):
    """More requests than slots and pages: admission waits for pages, prompts are cut at the budget."""
    cfg, t = model
    prompts = [_ids(n, seed=10 + n) for n in (5, 70, 1, 33, 90, 20)]
    srv = PipelineServer(cfg, M.NamedSource(cfg, 0), device="cpu", batch=2, microbatches=2, max_seq=128,
                         prefill_budget=24, dtype=torch.float32, cache_tokens=64 * 3)
    outs = srv.generate(prompts, 5, eos_ids=())
    for p, o in zip(prompts, outs):
        want, gaps = P.greedy(cfg.to_dict(), t, p, 5)
        assert o == want, (len(p), gaps)
    assert len(srv.eng.pool.free) == 3  # everything was given back
    with pytest.raises(ValueError):
        srv.submit(_ids(121), 8)  # exceeds max_seq


def test_pipeline_generates(model):
    cfg, t = model
    prompts = torch.tensor([_ids(6, seed=s) for s in range(4)]).view(2, 2, 6)
    out = run_pipeline_generate(cfg, M.NamedSource(cfg, 0), prompts, 4, 0, 1, batch=2, microbatches=2, max_seq=64,
                                dtype=torch.float32)
    for i in range(4):
        want, gaps = P.greedy(cfg.to_dict(), t, prompts.view(4, 6)[i].tolist(), 4)
        assert out.permute(1, 2, 0).reshape(4, -1)[i].tolist() == want, gaps  # out: [new, micro-batch, row]


def test_reference_style_chain(tmp_path, model):
    """Two nodes of the TCP chain (ingress + head) pass one request through by hand."""
    import socket

    from llm_sharding_amd.utils.node_worker import NodeWorker
    cfg, t = model
    folder = D.write_random_checkpoint(cfg, str(tmp_path / "m"), seed=0)
    ports = []
    for _ in range(2):
        with socket.socket() as sk:
            sk.bind(("127.0.0.1", 0))
            ports.append(sk.getsockname()[1])
    nodes = [NodeWorker(f"tcp://*:{ports[i]}", f"tcp://127.0.0.1:{ports[1 - i]}", i == 0, folder, dtype=torch.float32,
                        max_batch=1, max_seq=128, verbose=False) for i in range(2)]
    try:
        nodes[0].load_shards(0, 2)
        nodes[1].load_shards(2, 6)
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


def test_placement_knows_the_layers():
    from llm_sharding_amd.parallel.scheduler import kv_slots_for_memory, plan_stages, scratch_bytes, stage_memory
    cfg = get_preset("deretar-4k")
    plan = plan_stages(cfg, 4, kv_tokens=4096 * 32)
    assert [s.n_layers for s in plan.stages] == [8, 8, 8, 8]
    assert kv_slots_for_memory(cfg, 8, 4096, 288e9, plan.stages[0].weight_bytes) == 128
    m = stage_memory(cfg, 8, slots=32, max_seq=4096, prefill_rows=2048)
    assert m["kv"] == 8 * 32 * 4096 * 576 * 2 and m["scratch"] == scratch_bytes(cfg, 2048)


def test_trace_replay_needs_a_gpu(tmp_path):
    if torch.cuda.is_available():
        pytest.skip("a GPU is there")
    folder = D.write_random_checkpoint(M.stack(), str(tmp_path / "m"))
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", "float32",
                        "--out", str(tmp_path), "--max-tokens", "64"], stdin=subprocess.DEVNULL, capture_output=True,
                       text=True, timeout=100)
    assert r.returncode == 1 and "no GPU" in r.stderr


# ------------------------------------------------------------------------------ the oracle notices
def _mistakes():
    def off_by_one(qn, qr, kn, kr, v, scale):  # a row does not see itself (but the first)
        n = qn.shape[0]
        out = P_softmax(qn, qr, kn, kr, v, scale)
        return torch.cat([out[:1], out[:-1]]) if n > 1 else out

    P_softmax = P.softmax_heads
    return {
        "softmax_heads": off_by_one,
        "rotate": lambda x, pos, base, dims: x,
        "centred_norm": lambda x, w, eps: P.rms(x, eps) * w,
        "gain_norm": lambda x, w, eps: x * w,
        "clipped_glu": lambda a, b, limit: a * torch.sigmoid(1.702 * a) * (b + 1),
        "owner": lambda layers, i: i if layers[i].get("weights_of") is None else 5,
    }


@pytest.mark.parametrize("name", ["softmax_heads", "rotate", "centred_norm", "gain_norm", "clipped_glu", "owner"])
def test_a_planted_mistake_shows(model, name, monkeypatch):
    cfg, t = model
    ids = _ids(70)
    good = P.run(cfg.to_dict(), t, ids)
    monkeypatch.setattr(P, name, _mistakes()[name])
    try:
        bad = P.run(cfg.to_dict(), t, ids)
    except (KeyError, RuntimeError):
        return  # the mistake does not even fit the tensors
    assert M.rel(bad, good) > 0.1
