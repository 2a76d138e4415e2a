"""Config-driven layer stacks: a decoder described layer by layer instead of by one set of sizes.

A :class:`StackConfig` lists the layers in order; each :class:`LayerSpec` names its mixer and its
feed-forward with every size and constant of its own and how they are arranged around the residual
stream, and may use the tensors of another layer (``owner``, with a cache of its own) or another
layer's cached keys and values (``AttentionSpec.kv_from``). Designs (``models/deretar.py``,
``models/gupuvik.py``) only translate their config.json and tensor names into this description; the
mechanisms and their constants are parameters here, so that another design can combine them
differently.

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

    state_bytes = 0

    @property
    def scratch_width(self) -> int:
        """Values per row that a forward keeps besides the stream (every intermediate of the mixer)."""
        return self.q_rank * 2 + self.kv_rank + self.rot_dim + self.heads * (2 * self.dvp + self.dkp + self.rp)

    def part_bytes(self, items: int, elem_bytes: int) -> int:
        """Split partials of ``items`` (row, key split) pairs."""
        return items * self.heads * ((self.krp + 2) * 4 + self.cache_width * elem_bytes)

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

    def scratch_width(self, width: int) -> int:
        return self.ff

    def params(self, width: int) -> int:
        return 3 * self.ff * width

    active_params = params


def pad_part(n: int) -> int:
    """A head part as the attention kernels lay it out: 64 / 128 / 256 for the MFMA kernels, whole
    64s beyond (csrc/kernels/paged_attn.h)."""
    for k in (64, 128, 256):
        if n <= k:
            return k
    return pad_to(n, 64)


@dataclass(frozen=True)
class AttentionSpec:
    """Grouped-query softmax attention over a paged cache: query head h reads key / value head
    h / (heads / kv_heads). A row at position i sees the last ``window`` keys up to its own (0: all) and
    the first ``keep_first`` ones. Scores are q . k * scale, times a number per head (``head_temp``),
    then ``softcap`` tanh(. / softcap) (0: as they are); ``head_gate``: every head's output is multiplied by
    the sigmoid of one projected number."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: float = 0.0
    window: int = 0
    keep_first: int = 0
    bias: bool = False               # q, k and v projections have one
    head_temp: bool = False
    head_gate: bool = False
    kv_from: Optional[int] = None    # the layer whose cached keys and values this one reads

    def __post_init__(self):
        if min(self.heads, self.kv_heads, self.dim, self.vdim) < 1 or self.heads % self.kv_heads:
            raise ValueError(f"attention: bad sizes: {self}")
        if self.window < 0 or self.keep_first < 0 or self.softcap < 0:
            raise ValueError(f"attention: window, keep_first and softcap must not be negative: {self}")

    @property
    def group(self) -> int:
        return self.heads // self.kv_heads

    @property
    def dkp(self) -> int:
        return pad_part(self.dim)

    @property
    def dvp(self) -> int:
        return pad_part(self.vdim)

    @property
    def cache_width(self) -> int:
        """Values per token in this layer's cache (0: it reads another layer's)."""
        return 0 if self.kv_from is not None else self.kv_heads * (self.dkp + self.dvp)

    @property
    def state_bytes(self) -> int:
        return 0

    @property
    def scratch_width(self) -> int:
        own = self.kv_heads * (self.dkp + self.dvp) if self.kv_from is None else 0
        return self.heads * (self.dkp + self.dvp) + own + pad_to(self.heads, 16)

    def part_bytes(self, items: int, elem_bytes: int) -> int:
        return items * self.heads * (self.dvp + 2) * 4

    def params(self, width: int) -> int:
        n = self.heads * self.dim * (width + self.bias) + self.heads * self.vdim * width
        if self.kv_from is None:
            n += self.kv_heads * (self.dim + self.vdim) * (width + self.bias)
        return n + self.heads * self.head_temp + self.heads * width * self.head_gate


@dataclass(frozen=True)
class DeltaSpec:
    """Gated delta rule with one decay per head and key channel: per head a state S [dim, vdim],

        S <- g * S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q

    q, k (kv_heads of them) and v (heads) pass a causal convolution of ``taps`` tokens per channel and
    silu; q and k become unit vectors (``unit_eps`` inside the root), q times ``q_scale``. The decay and
    the output gate are projections of rank ``decay_rank`` / ``gate_rank``."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int
    decay_rank: int
    gate_rank: int
    q_scale: float
    unit_eps: float

    def __post_init__(self):
        if min(self.heads, self.kv_heads, self.dim, self.vdim, self.taps, self.decay_rank, self.gate_rank) < 1 \
                or self.heads % self.kv_heads:
            raise ValueError(f"delta rule: bad sizes: {self}")

    cache_width = 0

    @property
    def group(self) -> int:
        return self.heads // self.kv_heads

    @property
    def channels(self) -> int:
        """Convolved channels: q, k and v."""
        return 2 * self.kv_heads * self.dim + self.heads * self.vdim

    @property
    def state_dims(self) -> tuple:
        """(key channels, value channels) of a head's state as stored (csrc/kernels/delta.h)."""
        return tuple(next((k for k in (32, 64, 128) if n <= k), n) for n in (self.dim, self.vdim)) \
            if max(self.dim, self.vdim) <= 128 else (self.dim, self.vdim)

    @property
    def state_bytes(self) -> int:
        """Per sequence: the fp32 state and the convolutions' last inputs."""
        dk, dv = self.state_dims
        return 4 * (self.heads * dk * dv + self.taps * self.channels)

    @property
    def scratch_width(self) -> int:
        return self.channels + pad_to(self.decay_rank, 16) + pad_to(self.gate_rank, 16) \
            + self.heads * (2 * self.vdim + 2 * self.dim) + 2 * pad_to(self.heads, 16) + 256

    def part_bytes(self, items: int, elem_bytes: int) -> int:
        return 0

    def params(self, width: int) -> int:
        H, c = self.heads, self.channels
        low = self.decay_rank * (width + H * self.dim) + self.gate_rank * (width + H * self.vdim)
        return c * (width + self.taps) + H * width + low + H + H * self.dim + self.vdim + H * self.vdim * width


@dataclass(frozen=True)
class DenseSpec:
    """W_down act(W_up h), act the tanh form of gelu."""
    ff: int

    def __post_init__(self):
        if self.ff < 1:
            raise ValueError("feed-forward: ff must be positive")

    def scratch_width(self, width: int) -> int:
        return self.ff + 128

    def params(self, width: int) -> int:
        return 2 * self.ff * width

    active_params = params


@dataclass(frozen=True)
class MoeSpec:
    """``experts`` gated feed-forwards (silu) of which a token uses the ``top`` with the largest router
    logits, weighted by the softmax over these."""
    experts: int
    top: int
    ff: int

    def __post_init__(self):
        if min(self.experts, self.top, self.ff) < 1 or self.top > self.experts:
            raise ValueError(f"experts: bad sizes: {self}")

    def scratch_width(self, width: int) -> int:
        return 2 * pad_to(self.experts, 16) + self.top * (pad_to(self.ff, 128) + 2 * pad_to(width, 128) + 8)

    def params(self, width: int) -> int:
        return self.experts * (3 * self.ff + 1) * width

    def active_params(self, width: int) -> int:
        """Weights one token uses."""
        return (3 * self.ff * self.top + self.experts) * width


# How a layer's sublayers meet the residual stream
POST_NORM = "post_norm"  # each sublayer reads the stream; its result is normed, scaled per element and added
PARALLEL = "parallel"    # both read one norm of the stream; each result is added through a sigmoid gate per element


@dataclass(frozen=True)
class LayerSpec:
    mixer: Any  # LatentSpec | AttentionSpec | DeltaSpec
    mlp: Any    # GluSpec | DenseSpec | MoeSpec | None
    owner: int  # the layer whose tensors this one uses (itself unless it shares another's)
    block: str = POST_NORM


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

    def layer_params(self, i: int, active: bool = False) -> int:
        """Weights of layer i; ``active``: those that one token uses."""
        s, W = self.layers[i], self.hidden_size
        if s.block == PARALLEL:
            n = s.mixer.params(W) + 1 + W * W + W
            extra = W * W + W
        else:
            n, extra = s.mixer.params(W) + 2 * W, 2 * W
        if s.mlp is None:
            return n
        return n + extra + (s.mlp.active_params(W) if active else s.mlp.params(W))

    def layer_bytes(self, elem_bytes: int = 2) -> int:
        """The largest layer (placement is by whole layers)."""
        return max(self.layer_params(i) for i in range(self.num_hidden_layers)) * elem_bytes

    def layer_costs(self, elem_bytes: int = 2) -> list:
        """Bytes streamed per decode token, layer by layer."""
        return [float(self.layer_params(i, active=True) * elem_bytes + 2 * s.mixer.state_bytes)
                for i, s in enumerate(self.layers)]

    def stage_cuts(self) -> list:
        """Layer indices a pipeline stage may start at: a layer that reads another's keys and values
        runs on the stage that holds them."""
        tied = set()
        for i, s in enumerate(self.layers):
            j = getattr(s.mixer, "kv_from", None)
            if j is not None:
                tied.update(range(j + 1, i + 1))
        return [i for i in range(self.num_hidden_layers) if i not in tied]

    def kv_bytes_per_token_per_layer(self, elem_bytes: int = 2) -> int:
        return max(l.mixer.cache_width for l in self.layers) * elem_bytes

    def state_bytes_per_slot(self) -> int:
        """State a sequence carries besides its cache, the largest layer."""
        return max(l.mixer.state_bytes for l in self.layers)

    def scratch_bytes(self, rows: int, elem_bytes: int = 2) -> int:
        """What a stage engine allocates besides weights and cache for ``rows`` rows (the largest layer
        sets every buffer): StackEngine._scratch_set."""
        W = pad_to(self.hidden_size, 128)
        n = rows * (self.hidden_size * 4 + W * (4 + elem_bytes) + 12)
        inter = part = 0
        for l in self.layers:
            gates = 2 * pad_to(self.hidden_size, 16) if l.block == PARALLEL else 0
            inter = max(inter, l.mixer.scratch_width + gates
                        + (l.mlp.scratch_width(self.hidden_size) if l.mlp is not None else 0) + 5 * 128)
            part = max(part, l.mixer.part_bytes(1024, elem_bytes))
        return n + rows * inter * elem_bytes + part + (1 << 26) + 2 * 256 * 256 * 256 * 4

    def stream_bytes(self) -> int:
        """Bytes of one row of the residual stream between pipeline stages (fp32)."""
        return 4 * self.hidden_size

    def to_dict(self) -> dict:
        if self.raw is None:
            raise ValueError("this configuration was not read from a config.json")
        return self.raw


__all__ = ["StackConfig", "LayerSpec", "LatentSpec", "AttentionSpec", "DeltaSpec", "GluSpec", "DenseSpec", "MoeSpec",
           "POST_NORM", "PARALLEL", "pad_to", "pad_part"]
