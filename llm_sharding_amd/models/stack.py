"""Config-driven layer stacks: a decoder described layer by layer instead of by one set of sizes.

A :class:`StackConfig` lists the layers in order; each :class:`LayerSpec` names its mixer and its
feed-forward with every size and constant of its own, and may use the tensors of another layer
(``weights_of``) while keeping a cache of its own. Designs (``models/deretar.py``) only translate
their config.json and tensor names into this description; the mechanisms and their constants are
parameters here, so that another design can combine them differently.

:class:`StackConfig` also answers what the rest of the framework asks of a model configuration
(:class:`..config.LlamaConfig`): sizes for placement, cache sizing and the head.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, List, Optional


def pad_to(n: int, m: int) -> int:
    return -(-n // m) * m


@dataclass(frozen=True)
class LatentSpec:
    """Latent attention with a latent query, a shared rotated key part and an output gate."""
    heads: int
    dim: int        # unrotated query / key dimensions per head
    rot_dim: int    # rotated part: per head for the query, one for all heads for the key
    vdim: int
    kv_rank: int
    q_rank: int
    rot_base: float
    rot_dims: int   # leading entries of the rotated part that turn (rotate-half pairs)
    scale: float

    def __post_init__(self):
        if min(self.heads, self.dim, self.rot_dim, self.vdim, self.kv_rank, self.q_rank) < 1:
            raise ValueError(f"latent attention: sizes must be positive: {self}")
        if self.rot_dims % 2 or not 2 <= self.rot_dims <= self.rot_dim:
            raise ValueError(f"latent attention: rot dims {self.rot_dims} must be even and at most {self.rot_dim}")

    # ---- padded sizes of the kernels (csrc/kernels/latent.h)
    @property
    def dkp(self) -> int:
        return pad_to(self.dim, 64)

    @property
    def rp(self) -> int:
        return pad_to(self.rot_dim, 64)

    @property
    def dvp(self) -> int:
        return pad_to(self.vdim, 64)

    @property
    def krp(self) -> int:
        for k in (64, 128, 256, 512):  # the tuned kernels' latent sizes
            if self.kv_rank <= k:
                return k
        return pad_to(self.kv_rank, 64)

    @property
    def cache_width(self) -> int:
        """Cached values per token and layer."""
        return self.krp + self.rp

    def params(self, width: int) -> int:
        q = self.q_rank * width + self.heads * (self.dim + self.rot_dim) * self.q_rank + self.q_rank
        kv = (self.kv_rank + self.rot_dim) * width + self.heads * (self.dim + self.vdim) * self.kv_rank + self.kv_rank
        return q + kv + 2 * self.heads * self.vdim * width


@dataclass(frozen=True)
class GluSpec:
    """Clipped gated unit: g = min(gate, limit), u = clamp(up, -limit, limit),
    g * sigmoid(alpha g) * (u + shift)."""
    ff: int
    limit: float
    alpha: float
    shift: float

    def __post_init__(self):
        if self.ff < 1 or not self.limit > 0:
            raise ValueError(f"gated unit: ff and limit must be positive: {self}")

    def params(self, width: int) -> int:
        return 3 * self.ff * width


@dataclass(frozen=True)
class LayerSpec:
    mixer: LatentSpec
    mlp: Optional[GluSpec]
    owner: int  # the layer whose tensors this one uses (itself unless it shares another's)


@dataclass
class StackConfig:
    hidden_size: int
    vocab_size: int
    layers: List[LayerSpec]
    norm_eps: float
    embed_scale: float = 1.0
    norm_offset: float = 0.0   # norms on the sublayers' outputs multiply by (offset + w)
    max_position_embeddings: int = 1 << 17
    bos_token_id: int = 1
    eos_token_id: Any = None
    model_type: str = "stack"
    name: str = "stack"
    tie_word_embeddings: bool = True
    raw: Optional[dict] = None  # the config.json it was read from

    is_gpt2 = False

    # ------------------------------------------------------------------ framework view
    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @property
    def rms_norm_eps(self) -> float:
        return self.norm_eps

    @property
    def num_attention_heads(self) -> int:
        return max(l.mixer.heads for l in self.layers)

    @property
    def head_rows(self) -> int:
        """Head rows as served (whole 128-column groups; padding never wins the argmax)."""
        return pad_to(self.vocab_size, 128)

    @property
    def eos_ids(self) -> list:
        e = self.eos_token_id
        if e is None:
            return []
        return list(e) if isinstance(e, (list, tuple)) else [int(e)]

    def layer_params(self, i: int) -> int:
        s, W = self.layers[i], self.hidden_size
        n = s.mixer.params(W) + 2 * W
        return n + (s.mlp.params(W) + 2 * W if s.mlp is not None else 0)

    def layer_bytes(self, elem_bytes: int = 2) -> int:
        """The largest layer (placement is by whole layers)."""
        return max(self.layer_params(i) for i in range(self.num_hidden_layers)) * elem_bytes

    def layer_costs(self, elem_bytes: int = 2) -> list:
        """Bytes streamed per decode token, layer by layer."""
        return [float(self.layer_params(i) * elem_bytes) for i in range(self.num_hidden_layers)]

    def kv_bytes_per_token_per_layer(self, elem_bytes: int = 2) -> int:
        return max(l.mixer.cache_width for l in self.layers) * elem_bytes

    def scratch_bytes(self, rows: int, elem_bytes: int = 2) -> int:
        """What a stage engine allocates besides weights and cache for ``rows`` rows (the largest layer
        sets every buffer): StackEngine._scratch_set."""
        W = pad_to(self.hidden_size, 128)
        n = rows * (self.hidden_size * 4 + W * (4 + elem_bytes) + 12)
        inter = part = 0
        for l in self.layers:
            m = l.mixer
            inter = max(inter, m.q_rank * 2 + m.kv_rank + m.rot_dim + m.heads * (2 * m.dvp + m.dkp + m.rp)
                        + (l.mlp.ff if l.mlp is not None else 0) + 5 * 128)
            part = max(part, 1024 * m.heads * ((m.krp + 2) * 4 + m.cache_width * elem_bytes))
        return n + rows * inter * elem_bytes + part + (1 << 26) + 2 * 256 * 256 * 256 * 4

    def stream_bytes(self) -> int:
        """Bytes of one row of the residual stream between pipeline stages (fp32)."""
        return 4 * self.hidden_size

    def to_dict(self) -> dict:
        if self.raw is None:
            raise ValueError("this configuration was not read from a config.json")
        return self.raw


__all__ = ["StackConfig", "LayerSpec", "LatentSpec", "GluSpec", "pad_to"]
