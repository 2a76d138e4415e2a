"""Small Runidra models of the tests: layer lists, tensors under their checkpoint names, engines."""
import torch

from deretar_models import cut, feed, rel  # noqa: F401
from llm_sharding_amd.models import runidra as D
from llm_sharding_amd.runtime import registry as R
from llm_sharding_amd.runtime.engine import WeightSource


def stack(sharp=1.0):
    """Every branch: both mixers with each kind of feed-forward and without one, windows that do and do not divide a
    page, a loop behind the first layer, three streams, sizes that are no multiple of anything. ``sharp`` scales the
    scores: softmaxes that pick single keys show one that is missing or misplaced. (With a small eps the norm of matrix
    memory's read-outs would hide what they are divided by.)"""
    def att(heads, dim, rot, vdim, kv, q, size, mlp, base=500.0):
        return D.latent_entry(heads, dim, rot, vdim, kv, q, size, mlp, base, sharp * (dim + rot) ** -0.5)

    return D.make_config(88, 150, [
        D.mlstm_entry(3, 20, 28, D.dense(90), 6.0),
        att(5, 24, 16, 40, 48, 72, 37, D.moe(6, 2, 40, 50)),
        D.mlstm_entry(2, 36, 70, D.moe(5, 3, 20, 33)),
        att(18, 64, 32, 64, 128, 80, 64, None, 10000.0),
        att(1, 16, 8, 8, 200, 20, 100, D.dense(33), 77.0),
        D.mlstm_entry(4, 64, 32, None, 2.5),
    ], streams=3, loop=(1, 3, 2), eps=0.02, logit_scale=0.7, logit_softcap=9.0)


def tensors(cfg, seed=0):
    return D.random_tensors(cfg, seed)


def decided(cfg, seed=0):
    """As :func:`tensors`, without what bf16 activations turn into another result now and then: router biases are apart
    by more than logits can be (no close calls), and matrix memory's keys lie near its queries (no read-out of almost
    nothing, which its norm blows up)."""
    t = tensors(cfg, seed)
    for i, k in enumerate(sorted(t)):
        if k.endswith("mix.k"):
            t[k] = 0.5 * t[k] + t[k[:-1] + "q"]
        if k.endswith("router.b"):
            t[k] = (8.0 * torch.randperm(t[k].numel(), generator=torch.Generator().manual_seed(i))).to(t[k].dtype)
    return t


class NamedSource(WeightSource):
    """The tensors of :func:`tensors` (drawn on the CPU) on any device."""

    def __init__(self, cfg, seed=0, t=None):
        self.cfg, self.t = cfg, tensors(cfg, seed) if t is None else t

    def layer(self, i, device, dtype):
        p = f"l{self.cfg.layers[i].owner}."
        return {k[len(p):]: v.to(device, dtype) for k, v in self.t.items() if k.startswith(p)}

    def embedding(self, device, dtype):
        return self.t["embed"].to(device, dtype)

    def final_norm(self, device, dtype):
        return self.t["final.norm"].to(device, dtype)

    def lm_head(self, device, dtype):
        return self.t["head"].to(device, dtype)


def engine(cfg, device, dtype, seed=0, start=0, end=None, t=None, **kw):
    end = cfg.num_hidden_layers if end is None else end
    kw = {"max_slots": 4, "max_seq": 512, "max_prefill_rows": 512, **kw}
    return R.make_engine(cfg, start, end, device, dtype, has_embed=start == 0, has_head=end == cfg.num_hidden_layers,
                         source=NamedSource(cfg, seed, t), **kw)


LOUD, ASK = 148, 149  # tokens of :func:`asking`


def asking(window, heads=3, dim=24, rot=8, vdim=20, kv=40, q=32, eps=1e-5):
    """One layer of windowed attention whose token ASK attends to a LOUD token, if it sees one, and to little else: the
    tokens' embeddings have entries of their own that the projections turn into a latent and a query that meet."""
    cfg = D.make_config(72, 150, [D.latent_entry(heads, dim, rot, vdim, kv, q, window)], streams=2, eps=eps, logit_softcap=50.0)
    t = tensors(cfg)
    t["embed"][:, :2] = 0
    t["embed"][LOUD, 0] = t["embed"][ASK, 1] = 30.0
    for k, c in (("dkv", 0), ("dq", 1)):  # entry c alone feeds the latent's entry 0
        w = t[f"l0.mix.{k}"]
        w[0] = 0
        w[:, :2] = 0
        w[0, c] = 6.0
        t[f"l0.mix.{k}.norm"][0] = 1.0
    uk, uq = t["l0.mix.uk"].view(heads, dim, kv), t["l0.mix.uq"].view(heads, dim + rot, q)
    uk[:, 0], uq[:, 0] = 0, 0
    uk[:, :, 0], uq[:, :, 0] = 0, 0
    uk[:, 0, 0], uq[:, 0, 0] = 3.0, 3.0
    return cfg, t
