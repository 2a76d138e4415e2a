"""Small Gupuvik models of the tests: layer lists, tensors under their checkpoint names, engines."""
import torch

from deretar_models import cut, feed, rel  # noqa: F401
from llm_sharding_amd.models import gupuvik as G
from llm_sharding_amd.runtime import registry as R
from llm_sharding_amd.runtime.engine import WeightSource

RANK = 11


def stack(sharp=1.0):
    """Every branch: both mixers in turn, keys read from an earlier layer through another window, all three
    kinds of feed-forward (and none), grouped and single heads, sizes that are no multiple of anything.
    ``sharp`` scales the scores: softmaxes that pick single keys show one that is missing or misplaced."""
    def att(heads, kv, dim, vdim, size, keep, mlp, **kw):
        return G.attention_entry(heads, kv, dim, vdim, size, keep, mlp, scale=sharp * dim ** -0.5, **kw)

    return G.make_config(88, 150, [
        G.delta_entry(6, 2, 20, 24, 3, G.moe(5, 2, 40)),
        att(6, 3, 24, 40, 37, 3, G.dense(90), softcap=20.0),
        att(6, 3, 24, 40, 70, 0, G.moe(3, 3, 20), softcap=9.0, kv_from=1),
        G.delta_entry(2, 2, 36, 70, 5, None),
        att(5, 1, 72, 16, 9, 70, None),
        att(6, 3, 24, 40, 500, 2, G.moe(4, 1, 33), kv_from=1),
        G.delta_entry(3, 1, 33, 129, 2, G.dense(50)),
    ], eps=1e-5, embed_scale=1.7, rank=RANK)


def tensors(cfg, seed=0):
    return G.random_tensors(cfg, seed)


class NamedSource(WeightSource):
    """The tensors of :func:`tensors` (drawn on the CPU) on any device."""

    def __init__(self, cfg, seed=0):
        self.t = tensors(cfg, seed)

    def layer(self, i, device, dtype):
        p = f"l{i}."
        return {k[len(p):]: v.to(device, dtype) for k, v in self.t.items() if k.startswith(p)}

    def embedding(self, device, dtype):
        return self.t["embed"].to(device, dtype)

    def final_norm(self, device, dtype):
        return self.t["final.norm"].to(device, dtype)

    def lm_head(self, device, dtype):
        return self.t["head"].to(device, dtype)


def engine(cfg, device, dtype, seed=0, start=0, end=None, **kw):
    end = cfg.num_hidden_layers if end is None else end
    kw = {"max_slots": 4, "max_seq": 512, "max_prefill_rows": 512, **kw}
    return R.make_engine(cfg, start, end, device, dtype, has_embed=start == 0, has_head=end == cfg.num_hidden_layers,
                         source=NamedSource(cfg, seed), **kw)


def rel_most(got, want, rows=0.02):
    """As :func:`rel` without the worst few rows: bf16 activations now and then turn a router's close call, and
    a row with another expert is another result."""
    d = (got.double() - want.double())
    err = (d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt()
    keep = err.sort().values[:max(1, int(err.numel() * (1 - rows)))]
    w = want.double() - want.double().mean(-1, keepdim=True)
    return float(keep.max() / w.pow(2).mean(-1).sqrt().mean())
