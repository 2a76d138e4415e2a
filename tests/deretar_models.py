"""Small Deretar models of the tests: layer lists, tensors under their checkpoint names, engines."""
import torch

from llm_sharding_amd.models import deretar as D
from llm_sharding_amd.runtime import registry as R

MID = dict(heads=5, dim=40, rot_dim=24, vdim=56, kv_rank=48, q_rank=72, limit=1.25, base=500.0)
WIDE = dict(heads=18, dim=64, rot_dim=32, vdim=64, kv_rank=128, q_rank=80, limit=2.5)
LONE = dict(heads=1, dim=16, rot_dim=8, vdim=8, kv_rank=200, q_rank=20, rot_dims=6, limit=0.75, base=77.0)


def stack(sharp=1.0):
    """Layers of three sizes: shared tensors in a later and in an earlier direction, layers without a
    feed-forward, part of a rotated vector unturned. ``sharp`` scales the scores: softmaxes that pick
    single keys show a key that is missing or misplaced."""
    def e(d, ff, **kw):
        return D.layer_entry(ff=ff, scale=sharp * (d["dim"] + d["rot_dim"]) ** -0.5, **{**d, **kw})

    return D.make_config(88, 150, [e(MID, 90), e(WIDE, None), e(MID, 90, weights_of=0), e(LONE, 33),
                                   e(WIDE, None, weights_of=1), e(WIDE, 130)], eps=1e-5, embed_scale=6.5)


def tensors(cfg, seed=0, dtype=torch.bfloat16):
    t = {"embed": D.random_embedding(cfg, dtype, seed=seed), "final.norm": D.random_final_norm(cfg, dtype, seed=seed)}
    for i, s in enumerate(cfg.layers):
        if s.owner == i:
            t.update({f"l{i}.{k}": v for k, v in D.random_layer(cfg, i, dtype, seed=seed).items()})
    return t


class NamedSource(R.random_source(stack()).__class__):
    """The tensors of :func:`tensors` (drawn on the CPU) on any device."""

    def layer(self, i, device, dtype):
        return {k: v.to(device, dtype) for k, v in D.random_layer(self.cfg, i, torch.bfloat16, "cpu", self.seed).items()}

    def embedding(self, device, dtype):
        return D.random_embedding(self.cfg, torch.bfloat16, "cpu", self.seed).to(device, dtype)

    def final_norm(self, device, dtype):
        return D.random_final_norm(self.cfg, torch.bfloat16, "cpu", self.seed).to(device, dtype)

    lm_head = embedding


def engine(cfg, device, dtype, seed=0, start=0, end=None, **kw):
    end = cfg.num_hidden_layers if end is None else end
    kw = {"max_slots": 4, "max_seq": 512, "max_prefill_rows": 512, **kw}
    return R.make_engine(cfg, start, end, device, dtype, has_embed=start == 0, has_head=end == cfg.num_hidden_layers,
                         source=NamedSource(cfg, seed), **kw)


def feed(eng, parts):
    """One step of [(slot, tokens)] -> logits of all its rows."""
    slots, counts = [s for s, _ in parts], [len(t) for _, t in parts]
    slot, pos = eng.prefill_rows(slots, counts)
    h = eng.forward(eng.embed(torch.tensor([x for _, t in parts for x in t])), slot, pos)
    eng.advance(slots, counts)
    return eng.logits(h).cpu()


def cut(ids, sizes):
    """ids in portions of cycling sizes."""
    out, i, k = [], 0, 0
    while i < len(ids):
        out.append(ids[i:i + sizes[k % len(sizes)]])
        i, k = i + len(out[-1]), k + 1
    return out


def rel(got, want):
    """Worst row: root mean square of the difference over that of the wanted row's spread."""
    d = got.double() - want.double()
    w = want.double() - want.double().mean(-1, keepdim=True)
    return float((d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt().max() / w.pow(2).mean(-1).sqrt().mean())
