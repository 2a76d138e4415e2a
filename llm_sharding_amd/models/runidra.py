"""The Runidra design: config.json keys, tensor names, weight sources.

A decoder-only stack on several residual streams (hyper-connections): each sublayer reads a norm of a weighted sum of
them, and a matrix and the sublayer's result make every stream anew. A stretch of layers may run several times in a row
with the same tensors. Mixers: matrix memory (mLSTM); windowed latent attention with a sink and interleaved rotary pairs.
Feed-forwards: a gated unit with biases (gelu), experts with a gated shared one, or none. On disk: one folder with
``config.json`` (``"architecture": "Runidra"``) and ``model.safetensors``:

    embed / head [vocab, width]   final.norm [width]
    l<i>.norm1 [width]   l<i>.hc1.in / .out [streams]  .hc1.mix [streams, streams] (from, to)   (2 with a feed-forward)
  mlstm
    l<i>.mix.q / k [heads dim, width]  .v / .g [heads vdim, width]  .i / .f [heads, width]  .i.b / .f.b [heads]
    l<i>.mix.norm [heads vdim]  .o [width, heads vdim]
  latent_attention
    l<i>.mix.dq [q_rank, width]  .dq.norm  .uq [heads (dim + rot_dim), q_rank]
    l<i>.mix.dkv [kv_rank + rot_dim, width]  .dkv.norm  .uk [heads dim, kv_rank]  .uv [heads vdim, kv_rank]
    l<i>.mix.sink [heads]  .o [width, heads vdim]
  feed-forward
    l<i>.mlp.gate / up [ff, width]  .down [width, ff]  .gate.b / .up.b / .down.b
    l<i>.mlp.router [experts, width]  .router.b  .e<j>.gate / up / down  .shared.gate / up / down  .shared.sg [1, width]
"""
from __future__ import annotations

import json
import os
from typing import Optional

import torch

from .stack import HYPER, GluSpec, LatentSpec, LayerSpec, MlstmSpec, MoeSpec, StackConfig

ARCHITECTURE = "Runidra"
TIED_HEAD = False


def _mlstm(m: dict) -> MlstmSpec:
    dim = int(m["dim"])
    return MlstmSpec(heads=int(m["heads"]), dim=dim, vdim=int(m["vdim"]), gate_cap=float(m["gate_cap"]), q_scale=dim ** -0.5)


def _latent(m: dict) -> LatentSpec:
    window = int(m["mask"]["size"])
    if window < 1:
        raise ValueError(f"a window holds at least one token, not {window}")
    return LatentSpec(heads=int(m["heads"]), dim=int(m["dim"]), rot_dim=int(m["rot_dim"]), vdim=int(m["vdim"]),
                      kv_rank=int(m["kv_rank"]), q_rank=int(m["q_rank"]), rot_base=float(m["rot"]["base"]),
                      rot_dims=int(m["rot"]["dims"]), scale=float(m["scale"]), gate=False, window=window, sink=True,
                      interleaved=True)


MIXERS = {"mlstm": _mlstm, "latent_attention": _latent}


def _mlp(m: Optional[dict]):
    if m is None:
        return None
    if m.get("kind") == "dense":
        return GluSpec(ff=int(m["ff"]), gelu=True, bias=True)
    if m.get("kind") != "moe":
        raise ValueError(f"unknown feed-forward kind {m.get('kind')!r}")
    return MoeSpec(experts=int(m["router"]["experts"]), top=int(m["router"]["top"]), ff=int(m["expert"]["ff"]), bias=True,
                   shared_ff=int(m["shared"]["ff"]), shared_gate=True)


def config_from_dict(d: dict, name: str = "runidra", shapes: Optional[dict] = None) -> StackConfig:
    """``shapes`` (of a checkpoint's tensors) is not needed: config.json has every size."""
    entries = []
    for i, e in enumerate(d["layers"]):
        if e.get("type") not in MIXERS:
            raise ValueError(f"layer {i}: unknown mixer type {e.get('type')!r}")
        entries.append(LayerSpec(MIXERS[e["type"]](e["mixer"]), _mlp(e.get("mlp")), i, HYPER))
    streams, loop = int(d["streams"]), d.get("loop")
    if not entries or streams < 1:
        raise ValueError("a stack needs at least one layer and one stream")
    layers = entries
    if loop:
        start, stop, times = (int(loop[k]) for k in ("start", "stop", "times"))
        if not 0 <= start < stop <= len(entries) or times < 1:
            raise ValueError(f"bad loop {loop}")
        layers = entries[:start] + entries[start:stop] * times + entries[stop:]
    cap = float(d.get("logit_softcap") or 0.0)
    if cap < 0:
        raise ValueError("logit_softcap must not be negative")
    return StackConfig(hidden_size=int(d["width"]), vocab_size=int(d["vocab"]), layers=layers, norm_eps=float(d["norm"]["eps"]),
                       model_type="runidra", name=str(d.get("name", name)), tie_word_embeddings=TIED_HEAD, streams=streams,
                       logit_scale=float(d.get("logit_scale", 1.0)), logit_softcap=cap, raw=d)


def make_config(width: int, vocab: int, layers: list, streams: int = 2, loop: Optional[tuple] = None, eps: float = 1e-6,
                logit_scale: float = 1.0, logit_softcap: float = 30.0, name: str = "runidra") -> StackConfig:
    """A configuration from layer entries as config.json has them; ``loop``: (start, stop, times)."""
    d = {"architecture": ARCHITECTURE, "width": width, "vocab": vocab, "streams": streams, "norm": {"eps": eps},
         "logit_scale": logit_scale, "logit_softcap": logit_softcap, "layers": layers, "name": name}
    if loop is not None:
        d["loop"] = dict(zip(("start", "stop", "times"), loop))
    return config_from_dict(d)


def dense(ff: int) -> dict:
    return {"kind": "dense", "ff": ff}


def moe(experts: int, top: int, ff: int, shared: int) -> dict:
    return {"kind": "moe", "expert": {"ff": ff}, "shared": {"ff": shared}, "router": {"experts": experts, "top": top}}


def mlstm_entry(heads: int, dim: int, vdim: int, mlp: Optional[dict] = None, gate_cap: float = 15.0) -> dict:
    """One matrix memory entry of config.json's layer list."""
    return {"type": "mlstm", "mlp": mlp, "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": gate_cap}}


def latent_entry(heads: int, dim: int, rot_dim: int, vdim: int, kv_rank: int, q_rank: int, size: int, mlp: Optional[dict] = None,
                 base: float = 10000.0, scale: Optional[float] = None) -> dict:
    return {"type": "latent_attention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank,
                      "mask": {"size": size}, "rot": {"base": base, "dims": rot_dim},
                      "scale": (dim + rot_dim) ** -0.5 if scale is None else scale}}


# ------------------------------------------------------------------------------ tensors
def _mixer_shapes(m, W: int) -> dict:
    H = m.heads
    if isinstance(m, MlstmSpec):
        return {"q": (H * m.dim, W), "k": (H * m.dim, W), "v": (H * m.vdim, W), "g": (H * m.vdim, W), "i": (H, W), "i.b": (H,),
                "f": (H, W), "f.b": (H,), "norm": (H * m.vdim,), "o": (W, H * m.vdim)}
    return {"dq": (m.q_rank, W), "dq.norm": (m.q_rank,), "uq": (H * (m.dim + m.rot_dim), m.q_rank),
            "dkv": (m.kv_rank + m.rot_dim, W), "dkv.norm": (m.kv_rank,), "uk": (H * m.dim, m.kv_rank),
            "uv": (H * m.vdim, m.kv_rank), "sink": (H,), "o": (W, H * m.vdim)}


def _mlp_shapes(f, W: int) -> dict:
    if isinstance(f, GluSpec):
        return {"gate": (f.ff, W), "up": (f.ff, W), "down": (W, f.ff), "gate.b": (f.ff,), "up.b": (f.ff,), "down.b": (W,)}
    out = {"router": (f.experts, W), "router.b": (f.experts,), "shared.sg": (1, W)}
    for name, ff in [("shared", f.shared_ff)] + [(f"e{e}", f.ff) for e in range(f.experts)]:
        out.update({f"{name}.gate": (ff, W), f"{name}.up": (ff, W), f"{name}.down": (W, ff)})
    return out


def layer_shapes(cfg: StackConfig, i: int) -> dict:
    """Tensor shapes of layer run i (without their prefix)."""
    s, W, n = cfg.layers[i], cfg.hidden_size, cfg.streams
    out = {f"mix.{k}": v for k, v in _mixer_shapes(s.mixer, W).items()}
    if s.mlp is not None:
        out.update({f"mlp.{k}": v for k, v in _mlp_shapes(s.mlp, W).items()})
    for q in (1, 2) if s.mlp is not None else (1,):
        out.update({f"norm{q}": (W,), f"hc{q}.in": (n,), f"hc{q}.out": (n,), f"hc{q}.mix": (n, n)})
    return out


def _fill(k: str, t: torch.Tensor, g) -> torch.Tensor:
    """Random values of an ordinary size for tensor ``k``."""
    if k.endswith(("norm", "norm1", "norm2")):
        return t.uniform_(0.7, 1.3, generator=g)
    if ".hc" in k or k.startswith("hc"):
        if k.endswith("mix"):  # near the streams as they are
            return t.normal_(0.0, 0.2 / t.shape[0], generator=g).add_(torch.eye(t.shape[0], device=t.device), alpha=0.9)
        return t.uniform_(0.3, 1.0, generator=g)
    if k.endswith("mix.f.b"):  # memories of some to hundreds of tokens
        return t.uniform_(1.0, 6.0, generator=g)
    if k.endswith(".sink"):
        return t.normal_(0.0, 1.0, generator=g)
    if t.dim() == 1:
        return t.normal_(0.0, 0.3, generator=g)
    return t.normal_(0.0, t.shape[1] ** -0.5, generator=g)


def _draw(shapes: dict, salt: int, dtype, device, seed: int) -> dict:
    g = torch.Generator(device=device).manual_seed(seed * 100069 + salt)
    return {k: _fill(k, torch.empty(shp, dtype=torch.float32, device=device), g).to(dtype) for k, shp in shapes.items()}


def random_layer(cfg: StackConfig, i: int, dtype=torch.bfloat16, device="cpu", seed: int = 0) -> dict:
    """Deterministic random tensors of layer run i (those of its layer)."""
    return _draw(layer_shapes(cfg, i), 31 * cfg.layers[i].owner + 5, dtype, device, seed)


def random_embedding(cfg: StackConfig, dtype=torch.bfloat16, device="cpu", seed: int = 0) -> torch.Tensor:
    return _draw({"embed": (cfg.vocab_size, cfg.hidden_size)}, 7, dtype, device, seed)["embed"]


def random_head(cfg: StackConfig, dtype=torch.bfloat16, device="cpu", seed: int = 0) -> torch.Tensor:
    return _draw({"head": (cfg.vocab_size, cfg.hidden_size)}, 13, dtype, device, seed)["head"]


def random_final_norm(cfg: StackConfig, dtype=torch.bfloat16, device="cpu", seed: int = 0) -> torch.Tensor:
    return _draw({"final.norm": (cfg.hidden_size,)}, 11, dtype, device, seed)["final.norm"]


def random_tensors(cfg: StackConfig, seed: int = 0, dtype=torch.bfloat16) -> dict:
    """A whole random checkpoint, by tensor name."""
    t = {"embed": random_embedding(cfg, dtype, seed=seed), "head": random_head(cfg, dtype, seed=seed),
         "final.norm": random_final_norm(cfg, dtype, seed=seed)}
    for i, s in enumerate(cfg.layers):
        if f"l{s.owner}.norm1" not in t:
            t.update({f"l{s.owner}.{k}": v for k, v in random_layer(cfg, i, dtype, seed=seed).items()})
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


__all__ = ["ARCHITECTURE", "config_from_dict", "make_config", "mlstm_entry", "latent_entry", "dense", "moe", "layer_shapes",
           "random_layer", "random_embedding", "random_head", "random_final_norm", "random_tensors", "write_random_checkpoint"]
