"""The Deretar design: config.json keys, tensor names, weight sources.

A decoder-only stack of latent-attention layers with norms on the sublayers' outputs. On disk: one
folder with ``config.json`` (``"architecture": "Deretar"``) and ``model.safetensors``. Layer i's
tensors start with ``l<i>.``; a layer with ``weights_of`` has none of its own.

    embed [vocab, width]                 also the head (without the embedding scale)
    l<i>.norm1 / norm2 / ls1 / ls2 [width]
    l<i>.mix.dq [q_rank, width]  .dq.norm  .uq [heads (dim + rot_dim), q_rank]
    l<i>.mix.dkv [kv_rank + rot_dim, width]  .dkv.norm  .uk [heads dim, kv_rank]  .uv [heads vdim, kv_rank]
    l<i>.mix.g [heads vdim, width]  .o [width, heads vdim]
    l<i>.mlp.gate / up [ff, width]  .down [width, ff]
    final.norm [width]
"""
from __future__ import annotations

import json
import os
from typing import Optional

import torch

from .stack import GluSpec, LatentSpec, LayerSpec, StackConfig

ARCHITECTURE = "Deretar"
GLU_ALPHA, GLU_SHIFT = 1.702, 1.0   # fixed by the design
NORM_OFFSET = 1.0                   # norm weights are stored around zero
TIED_HEAD = True                    # the head is the embedding table


def _mixer(entry: dict) -> LatentSpec:
    if entry.get("type") != "latent_attention":
        raise ValueError(f"unknown mixer type {entry.get('type')!r}")
    m = entry["mixer"]
    return LatentSpec(heads=int(m["heads"]), dim=int(m["dim"]), rot_dim=int(m["rot_dim"]), vdim=int(m["vdim"]),
                      kv_rank=int(m["kv_rank"]), q_rank=int(m["q_rank"]), rot_base=float(m["rot"]["base"]),
                      rot_dims=int(m["rot"]["dims"]), scale=float(m["scale"]))


def _mlp(entry: dict) -> Optional[GluSpec]:
    m = entry.get("mlp")
    if m is None:
        return None
    if m.get("kind", "dense") != "dense":
        raise ValueError(f"unknown feed-forward kind {m.get('kind')!r}")
    if not float(m["limit"]) > 0:
        raise ValueError("gated unit: limit must be positive")
    return GluSpec(ff=int(m["ff"]), limit=float(m["limit"]), alpha=GLU_ALPHA, shift=GLU_SHIFT)


def config_from_dict(d: dict, name: str = "deretar", shapes: Optional[dict] = None) -> StackConfig:
    """``shapes`` (of a checkpoint's tensors) is not needed: config.json has every size."""
    entries = d["layers"]
    layers = []
    for i, e in enumerate(entries):
        j, seen = i, set()
        while entries[j].get("weights_of") is not None:
            seen.add(j)
            j = int(entries[j]["weights_of"])
            if not 0 <= j < len(entries) or j in seen:
                raise ValueError(f"layer {i}: weights_of leads to no layer with tensors")
        spec = LayerSpec(_mixer(e), _mlp(e), j)
        if j != i and (spec.mixer, spec.mlp) != (_mixer(entries[j]), _mlp(entries[j])):
            raise ValueError(f"layer {i} uses layer {j}'s tensors but is described differently")
        layers.append(spec)
    if not layers:
        raise ValueError("a stack needs at least one layer")
    return StackConfig(hidden_size=int(d["width"]), vocab_size=int(d["vocab"]), layers=layers,
                       norm_eps=float(d["norm"]["eps"]), embed_scale=float(d["embedding"]["scale"]),
                       norm_offset=NORM_OFFSET, model_type="deretar", name=str(d.get("name", name)), raw=d)


def make_config(width: int, vocab: int, layers: list, eps: float = 1e-6, embed_scale: Optional[float] = None,
                name: str = "deretar") -> StackConfig:
    """A configuration from layer entries as config.json has them."""
    d = {"architecture": ARCHITECTURE, "width": width, "vocab": vocab, "norm": {"eps": eps},
         "embedding": {"scale": float(width) ** 0.5 if embed_scale is None else embed_scale}, "layers": layers,
         "name": name}
    return config_from_dict(d)


def layer_entry(heads: int, dim: int, rot_dim: int, vdim: int, kv_rank: int, q_rank: int, ff: Optional[int] = None,
                limit: float = 7.0, base: float = 10000.0, rot_dims: Optional[int] = None,
                scale: Optional[float] = None, weights_of: Optional[int] = None) -> dict:
    """One entry of config.json's layer list."""
    e = {"type": "latent_attention",
         "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank,
                   "rot": {"base": base, "dims": rot_dim if rot_dims is None else rot_dims},
                   "scale": (dim + rot_dim) ** -0.5 if scale is None else scale},
         "mlp": None if ff is None else {"kind": "dense", "ff": ff, "limit": limit}}
    if weights_of is not None:
        e["weights_of"] = weights_of
    return e


# ------------------------------------------------------------------------------ tensors
def layer_shapes(cfg: StackConfig, i: int) -> dict:
    """Tensor shapes of layer i (without its prefix)."""
    s, W = cfg.layers[i], cfg.hidden_size
    m, H = s.mixer, s.mixer.heads
    out = {"norm1": (W,), "ls1": (W,), "mix.dq": (m.q_rank, W), "mix.dq.norm": (m.q_rank,),
           "mix.uq": (H * (m.dim + m.rot_dim), m.q_rank), "mix.dkv": (m.kv_rank + m.rot_dim, W),
           "mix.dkv.norm": (m.kv_rank,), "mix.uk": (H * m.dim, m.kv_rank), "mix.uv": (H * m.vdim, m.kv_rank),
           "mix.g": (H * m.vdim, W), "mix.o": (W, H * m.vdim)}
    if s.mlp is not None:
        out.update({"norm2": (W,), "ls2": (W,), "mlp.gate": (s.mlp.ff, W), "mlp.up": (s.mlp.ff, W),
                    "mlp.down": (W, s.mlp.ff)})
    return out


def random_layer(cfg: StackConfig, i: int, dtype=torch.bfloat16, device="cpu", seed: int = 0) -> dict:
    """Deterministic random tensors of layer i (of its owner, where it shares)."""
    i = cfg.layers[i].owner
    g = torch.Generator(device=device).manual_seed(seed * 100057 + 31 * i + 5)
    out = {}
    for k, shp in layer_shapes(cfg, i).items():
        t = torch.empty(shp, dtype=torch.float32, device=device)
        if k in ("norm1", "norm2"):
            t.normal_(0.0, 0.1, generator=g)
        elif k in ("ls1", "ls2"):
            t.uniform_(0.5, 1.5, generator=g)
        elif len(shp) == 1:
            t.uniform_(0.8, 1.2, generator=g)
        else:
            t.normal_(0.0, shp[1] ** -0.5, generator=g)
        out[k] = t.to(dtype)
    return out


def random_embedding(cfg: StackConfig, dtype=torch.bfloat16, device="cpu", seed: int = 0) -> torch.Tensor:
    g = torch.Generator(device=device).manual_seed(seed * 100057 + 7)
    t = torch.empty((cfg.vocab_size, cfg.hidden_size), dtype=torch.float32, device=device)
    return t.normal_(0.0, cfg.hidden_size ** -0.5, generator=g).to(dtype)


def random_final_norm(cfg: StackConfig, dtype=torch.bfloat16, device="cpu", seed: int = 0) -> torch.Tensor:
    g = torch.Generator(device=device).manual_seed(seed * 100057 + 11)
    return torch.empty(cfg.hidden_size, dtype=torch.float32, device=device).normal_(0.0, 0.1, generator=g).to(dtype)


def write_random_checkpoint(cfg: StackConfig, folder: str, seed: int = 0, dtype=torch.bfloat16) -> str:
    """config.json and model.safetensors of random tensors."""
    from safetensors.torch import save_file
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg.to_dict(), f, indent=1)
    t = {"embed": random_embedding(cfg, dtype, seed=seed), "final.norm": random_final_norm(cfg, dtype, seed=seed)}
    for i, s in enumerate(cfg.layers):
        if s.owner == i:
            t.update({f"l{i}.{k}": v for k, v in random_layer(cfg, i, dtype, seed=seed).items()})
    save_file({k: v.contiguous() for k, v in t.items()}, os.path.join(folder, "model.safetensors"))
    return folder


__all__ = ["ARCHITECTURE", "config_from_dict", "make_config", "layer_entry", "layer_shapes",
           "random_layer", "random_embedding", "random_final_norm", "write_random_checkpoint"]
