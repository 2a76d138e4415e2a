"""The Gupuvik design: config.json keys, tensor names, weight sources.

A decoder-only stack whose layers read one norm of the stream in parallel (mixer and feed-forward),
both results joining it through a sigmoid gate per element. Mixers are windowed attention (keeping the
first tokens; a layer may read an earlier layer's keys and values) or a gated delta rule with one
decay per key channel; feed-forwards are dense or a mixture of experts. On disk: one folder with
``config.json`` (``"architecture": "Gupuvik"``) and ``model.safetensors``:

    embed, head [vocab, width]   final.norm []
    l<i>.norm1 []   .rg1 [width, width]  .rg1.b [width]   (.rg2, .rg2.b with a feed-forward)
  attention
    l<i>.mix.q [heads dim, width]  .q.b   (.k, .k.b, .v, .v.b unless kv_from)   .temp [heads]
    l<i>.mix.g [heads, width]  .o [width, heads vdim]
  channel_delta
    l<i>.mix.q / k [kv_heads dim, width]  .v [heads vdim, width]  (.q.conv / .k.conv / .v.conv [channels, taps])
    l<i>.mix.b [heads, width]  .A_log [heads]  .dt_bias [heads dim]  .norm [vdim]
    l<i>.mix.a1 [r, width]  .a2 [heads dim, r]  .g1 [s, width]  .g2 [heads vdim, s]  .o [width, heads vdim]
  feed-forward
    l<i>.mlp.up [ff, width]  .down [width, ff]          dense
    l<i>.mlp.router [experts, width]  .e<j>.gate / up [ff, width]  .e<j>.down [width, ff]

The ranks r and s are not in config.json: the tensors' shapes give them.
"""
from __future__ import annotations

import json
import os
from typing import Optional

import torch

from .stack import PARALLEL, AttentionSpec, DeltaSpec, DenseSpec, LayerSpec, MoeSpec, StackConfig

ARCHITECTURE = "Gupuvik"
UNIT_EPS = 1e-6            # under the root of the delta rule's unit vectors; fixed by the design
TIED_HEAD = False


def _attention(m: dict) -> AttentionSpec:
    mask = m.get("mask") or {}
    return AttentionSpec(heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                         scale=float(m["scale"]), softcap=float(m.get("softcap") or 0.0),
                         window=int(mask.get("size") or 0), keep_first=int(mask.get("keep_first") or 0), bias=True,
                         head_temp=True, head_gate=True,
                         kv_from=None if m.get("kv_from") is None else int(m["kv_from"]))


def _delta(m: dict, i: int, shapes: Optional[dict], rank: Optional[int]) -> DeltaSpec:
    def r(name):
        if shapes is not None:
            return int(shapes[f"l{i}.mix.{name}"][0])
        return int(m["dim"]) if rank is None else rank

    return DeltaSpec(heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                     taps=int(m["conv"]), decay_rank=r("a1"), gate_rank=r("g1"), q_scale=float(m["dim"]) ** -0.5,
                     unit_eps=UNIT_EPS)


def _mlp(m: Optional[dict]):
    if m is None:
        return None
    kind = m.get("kind", "dense")
    if kind == "dense":
        return DenseSpec(ff=int(m["ff"]))
    if kind == "moe":
        return MoeSpec(experts=int(m["router"]["experts"]), top=int(m["router"]["top"]), ff=int(m["expert"]["ff"]))
    raise ValueError(f"unknown feed-forward kind {kind!r}")


def config_from_dict(d: dict, name: str = "gupuvik", shapes: Optional[dict] = None,
                     rank: Optional[int] = None) -> StackConfig:
    """``shapes``: tensor name -> shape of a checkpoint (the ranks of the decay and gate projections);
    without one the ranks are ``rank``, or the key size."""
    layers = []
    for i, e in enumerate(d["layers"]):
        kind, m = e.get("type"), e["mixer"]
        if kind == "attention":
            mixer = _attention(m)
        elif kind == "channel_delta":
            mixer = _delta(m, i, shapes, rank)
        else:
            raise ValueError(f"layer {i}: unknown mixer type {kind!r}")
        j = getattr(mixer, "kv_from", None)
        if j is not None:
            src = layers[j].mixer if 0 <= j < i else None
            if not isinstance(src, AttentionSpec) or src.kv_from is not None:
                raise ValueError(f"layer {i}: kv_from {j} is no earlier attention layer with keys of its own")
            if (src.kv_heads, src.dim, src.vdim) != (mixer.kv_heads, mixer.dim, mixer.vdim):
                raise ValueError(f"layer {i} reads layer {j}'s keys but has other sizes")
        layers.append(LayerSpec(mixer, _mlp(e.get("mlp")), i, PARALLEL))
    if not layers:
        raise ValueError("a stack needs at least one layer")
    return StackConfig(hidden_size=int(d["width"]), vocab_size=int(d["vocab"]), layers=layers,
                       norm_eps=float(d["norm"]["eps"]), embed_scale=float(d["embedding"]["scale"]),
                       model_type="gupuvik", name=str(d.get("name", name)), tie_word_embeddings=TIED_HEAD, raw=d)


def make_config(width: int, vocab: int, layers: list, eps: float = 1e-6, embed_scale: float = 1.0,
                name: str = "gupuvik", rank: Optional[int] = None) -> StackConfig:
    """A configuration from layer entries as config.json has them."""
    d = {"architecture": ARCHITECTURE, "width": width, "vocab": vocab, "norm": {"eps": eps},
         "embedding": {"scale": embed_scale}, "layers": layers, "name": name}
    return config_from_dict(d, rank=rank)


def dense(ff: int) -> dict:
    return {"kind": "dense", "ff": ff}


def moe(experts: int, top: int, ff: int) -> dict:
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}


def attention_entry(heads: int, kv_heads: int, dim: int, vdim: int, size: int, keep_first: int = 0,
                    mlp: Optional[dict] = None, scale: Optional[float] = None, softcap: float = 50.0,
                    kv_from: Optional[int] = None) -> dict:
    """One attention entry of config.json's layer list."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": size, "keep_first": keep_first},
         "scale": dim ** -0.5 if scale is None else scale, "softcap": softcap}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m, "mlp": mlp}


def delta_entry(heads: int, kv_heads: int, dim: int, vdim: int, conv: int = 4, mlp: Optional[dict] = None) -> dict:
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                                               "conv": conv}, "mlp": mlp}


# ------------------------------------------------------------------------------ tensors
def layer_shapes(cfg: StackConfig, i: int) -> dict:
    """Tensor shapes of layer i (without its prefix)."""
    s, W = cfg.layers[i], cfg.hidden_size
    m, H = s.mixer, s.mixer.heads
    out = {"norm1": (), "rg1": (W, W), "rg1.b": (W,)}
    if isinstance(m, AttentionSpec):
        parts = {"q": H * m.dim}
        if m.kv_from is None:
            parts.update({"k": m.kv_heads * m.dim, "v": m.kv_heads * m.vdim})
        for k, n in parts.items():
            out.update({f"mix.{k}": (n, W), f"mix.{k}.b": (n,)})
        out.update({"mix.temp": (H,), "mix.g": (H, W)})
    else:
        for k, n in (("q", m.kv_heads * m.dim), ("k", m.kv_heads * m.dim), ("v", H * m.vdim)):
            out.update({f"mix.{k}": (n, W), f"mix.{k}.conv": (n, m.taps)})
        out.update({"mix.b": (H, W), "mix.A_log": (H,), "mix.dt_bias": (H * m.dim,), "mix.norm": (m.vdim,),
                    "mix.a1": (m.decay_rank, W), "mix.a2": (H * m.dim, m.decay_rank), "mix.g1": (m.gate_rank, W),
                    "mix.g2": (H * m.vdim, m.gate_rank)})
    out["mix.o"] = (W, H * m.vdim)
    if s.mlp is not None:
        out.update({"rg2": (W, W), "rg2.b": (W,)})
    if isinstance(s.mlp, DenseSpec):
        out.update({"mlp.up": (s.mlp.ff, W), "mlp.down": (W, s.mlp.ff)})
    elif isinstance(s.mlp, MoeSpec):
        out["mlp.router"] = (s.mlp.experts, W)
        for e in range(s.mlp.experts):
            out.update({f"mlp.e{e}.gate": (s.mlp.ff, W), f"mlp.e{e}.up": (s.mlp.ff, W), f"mlp.e{e}.down": (W, s.mlp.ff)})
    return out


def _uniform(t, lo, hi, g):
    return t.uniform_(lo, hi, generator=g)


def random_layer(cfg: StackConfig, i: int, dtype=torch.bfloat16, device="cpu", seed: int = 0) -> dict:
    """Deterministic random tensors of layer i: decays from slow to fast, keys and gates of ordinary size."""
    g = torch.Generator(device=device).manual_seed(seed * 100057 + 31 * i + 5)
    out = {}
    for k, shp in layer_shapes(cfg, i).items():
        t = torch.empty(shp, dtype=torch.float32, device=device)
        if k in ("norm1", "mix.norm", "mix.temp"):
            _uniform(t, 0.8, 1.3, g)
        elif k == "mix.A_log":
            _uniform(t, -3.0, 1.0, g)
        elif k == "mix.dt_bias":
            _uniform(t, -4.0, 0.0, g)
        elif k.endswith(".conv"):
            t.normal_(0.0, shp[1] ** -0.5, generator=g)
        elif len(shp) == 1:
            t.normal_(0.0, 0.3, generator=g)
        else:
            t.normal_(0.0, shp[1] ** -0.5, generator=g)
        out[k] = t.to(dtype)
    return out


def _random_table(cfg: StackConfig, salt: int, std: float, dtype, device, seed: int) -> torch.Tensor:
    g = torch.Generator(device=device).manual_seed(seed * 100057 + salt)
    t = torch.empty((cfg.vocab_size, cfg.hidden_size), dtype=torch.float32, device=device)
    return t.normal_(0.0, std, generator=g).to(dtype)


def random_embedding(cfg: StackConfig, dtype=torch.bfloat16, device="cpu", seed: int = 0) -> torch.Tensor:
    return _random_table(cfg, 7, 1.0, dtype, device, seed)


def random_head(cfg: StackConfig, dtype=torch.bfloat16, device="cpu", seed: int = 0) -> torch.Tensor:
    return _random_table(cfg, 13, cfg.hidden_size ** -0.5, dtype, device, seed)


def random_final_norm(cfg: StackConfig, dtype=torch.bfloat16, device="cpu", seed: int = 0) -> torch.Tensor:
    g = torch.Generator(device=device).manual_seed(seed * 100057 + 11)
    return torch.empty((), dtype=torch.float32, device=device).uniform_(0.8, 1.3, generator=g).to(dtype)


def random_tensors(cfg: StackConfig, seed: int = 0, dtype=torch.bfloat16) -> dict:
    """A whole random checkpoint, by tensor name."""
    t = {"embed": random_embedding(cfg, dtype, seed=seed), "head": random_head(cfg, dtype, seed=seed),
         "final.norm": random_final_norm(cfg, dtype, seed=seed)}
    for i in range(cfg.num_hidden_layers):
        t.update({f"l{i}.{k}": v for k, v in random_layer(cfg, i, dtype, seed=seed).items()})
    return t


def write_random_checkpoint(cfg: StackConfig, folder: str, seed: int = 0, dtype=torch.bfloat16) -> str:
    """config.json and model.safetensors of random tensors."""
    from safetensors.torch import save_file
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg.to_dict(), f, indent=1)
    save_file({k: v.contiguous() for k, v in random_tensors(cfg, seed, dtype).items()},
              os.path.join(folder, "model.safetensors"))
    return folder


__all__ = ["ARCHITECTURE", "config_from_dict", "make_config", "attention_entry", "delta_entry", "dense", "moe",
           "layer_shapes", "random_layer", "random_embedding", "random_head", "random_final_norm", "random_tensors",
           "write_random_checkpoint"]
