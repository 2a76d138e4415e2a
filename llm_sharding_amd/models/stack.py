"""Config-driven layer stacks: a decoder described layer by layer instead of by one set of sizes.

A :class:`StackConfig` lists the layers in order; each :class:`LayerSpec` names its mixer and its
feed-forward with every size and constant of its own and how they are arranged around the residual
stream, and may use the tensors of another layer (``owner``, with a cache of its own) or another
layer's cached keys and values (``AttentionSpec.kv_from``). A stretch of layers that runs several times in
a row is listed once per run (``LayerSpec.enters`` marks where a pass begins). Designs
(``models/deretar.py``, ``gupuvik.py``, ``dumizen.py``, ``runidra.py``) only translate their config.json and tensor names
into this description; the mechanisms and their constants are parameters here, so that another design can
combine them differently.

:class:`StackConfig` also answers what the rest of the framework asks of a model configuration
(:class:`..config.LlamaConfig`): sizes for placement, cache sizing and the head.
"""
from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Any, List, Optional


def pad_to(n: int, m: int) -> int:
    return -(-n // m) * m


@dataclass(frozen=True)
class RotarySpec:
    """Rotary positions: pairs (i, i + dims / 2) of a head's first ``dims`` values turn by p * f_i,
    f_i = base^(-2i / dims). With ``factor`` (YaRN) pairs that turn fewer than ``slow`` times over ``original``
    positions are slowed by it, those of more than ``fast`` turns are kept, the others lie between; the
    rotated values grow by 0.1 ln(factor) + 1."""
    base: float
    dims: int
    factor: float = 0.0   # 0: no scaling
    original: float = 0.0
    fast: float = 0.0
    slow: float = 0.0

    def __post_init__(self):
        if self.dims % 2 or self.dims < 2 or self.base <= 1 or self.factor < 0 \
                or (self.factor and min(self.original, self.fast, self.slow) <= 0):
            raise ValueError(f"rotary positions: bad values: {self}")

    def frequencies(self) -> list:
        n, f = self.dims, [self.base ** (-2.0 * i / self.dims) for i in range(self.dims // 2)]
        if not self.factor:
            return f

        def at(turns):  # the pair index, times two, that turns so often over ``original`` positions
            return n * math.log(self.original / (2 * math.pi * turns)) / (2 * math.log(self.base))
        lo, hi = max(math.floor(at(self.fast)), 0), min(math.ceil(at(self.slow)), n - 1)
        ramp = [min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0) for i in range(n // 2)]
        return [x / self.factor * r + x * (1 - r) for x, r in zip(f, ramp)]

    @property
    def amplitude(self) -> float:
        return 0.1 * math.log(self.factor) + 1 if self.factor else 1.0


@dataclass(frozen=True)
class LatentSpec:
    """Latent attention with a latent query and a shared rotated key part. A row at position i sees the last
    ``window`` keys up to its own (0: all). ``gate``: every output value is multiplied by the sigmoid of a projected
    one; ``sink``: the softmax's denominator has one more term, exp of a number per head. Pairs of the rotated part
    are (i, i + rot_dims / 2), or ``interleaved`` (2i, 2i + 1)."""
    heads: int
    dim: int        # unrotated query / key dimensions per head
    rot_dim: int    # rotated part: per head for the query, one for all heads for the key
    vdim: int
    kv_rank: int
    q_rank: int
    rot_base: float
    rot_dims: int   # leading entries of the rotated part that turn
    scale: float
    gate: bool = True
    window: int = 0
    sink: bool = False
    interleaved: bool = False

    def __post_init__(self):
        if min(self.heads, self.dim, self.rot_dim, self.vdim, self.kv_rank, self.q_rank) < 1 or self.window < 0:
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
        return self.q_rank * 2 + self.kv_rank + self.rot_dim + self.heads * ((1 + self.gate) * self.dvp + self.dkp + self.rp)

    def part_bytes(self, items: int, elem_bytes: int) -> int:
        """Split partials of ``items`` (row, key split) pairs."""
        return items * self.heads * ((self.krp + 2) * 4 + self.cache_width * elem_bytes)

    def params(self, width: int) -> int:
        q = self.q_rank * width + self.heads * (self.dim + self.rot_dim) * self.q_rank + self.q_rank
        kv = (self.kv_rank + self.rot_dim) * width + self.heads * (self.dim + self.vdim) * self.kv_rank + self.kv_rank
        return q + kv + (1 + self.gate) * self.heads * self.vdim * width + self.sink * self.heads


@dataclass(frozen=True)
class GluSpec:
    """Gated unit act(gate) * up, act silu or with ``gelu`` the tanh form of gelu. With ``limit`` the clipped unit:
    g = min(gate, limit), u = clamp(up, -limit, limit), g * sigmoid(alpha g) * (u + shift). ``bias`` (with
    gelu): all three projections have one."""
    ff: int
    limit: float = 0.0
    alpha: float = 1.0
    shift: float = 0.0
    gelu: bool = False
    bias: bool = False

    def __post_init__(self):
        if self.ff < 1 or self.limit < 0 or (self.gelu and self.limit) or (self.bias and not self.gelu):
            raise ValueError(f"gated unit: bad values: {self}")

    def scratch_width(self, width: int) -> int:
        return pad_to(self.ff, 128)

    def params(self, width: int) -> int:
        return 3 * self.ff * width + self.bias * (2 * self.ff + width)

    active_params = params


def pad_part(n: int) -> int:
    """A head part as the attention kernels lay it out: 64 / 128 / 256 for the MFMA kernels, whole
    64s beyond (csrc/kernels/paged_attn.h)."""
    for k in (64, 128, 256):
        if n <= k:
            return k
    return pad_to(n, 64)


HEAD, WHOLE = "head", "whole"  # AttentionSpec.qk_norm: over each head's values / over the whole projection


@dataclass(frozen=True)
class AttentionSpec:
    """Grouped-query attention over a paged cache: query head h reads key / value head
    h / (heads / kv_heads). A row at position i sees the last ``window`` keys up to its own (0: all) and
    the first ``keep_first`` ones, and with ``pool`` beside the window one key and one value for every block
    of ``pool`` tokens that lies wholly behind it: the means of the block's cached keys and values.

    Queries and keys may be RMS-normed (``qk_norm``) and rotated (``rot``) first. Scores are q . k * scale,
    times a number per head (``head_temp``) and 1 + temp_coef ln(floor((p + 1) / temp_every) + 1) at position p,
    then ``softcap`` tanh(. / softcap) (0: as they are), less r1 ln(1 + r2 distance) per head
    (``distance_bias``). Weights are their softmax, with ``sink`` over one more score of 0 without a value; or
    with ``sigmoid`` each key's weight is the sigmoid of its score plus a number per head.

    ``head_gate``: every head's output is multiplied by the sigmoid of one projected number; ``elem_gate``:
    every output value by that of its own. ``tied_values``: the values are the keys as projected."""
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
    pool: int = 0
    qk_norm: Optional[str] = None    # HEAD | WHOLE
    rot: Optional[RotarySpec] = None
    temp_coef: float = 0.0
    temp_every: int = 1
    distance_bias: bool = False
    sigmoid: bool = False
    sink: bool = False
    elem_gate: bool = False
    tied_values: bool = False
    out_bias: bool = False

    def __post_init__(self):
        if min(self.heads, self.kv_heads, self.dim, self.vdim) < 1 or self.heads % self.kv_heads:
            raise ValueError(f"attention: bad sizes: {self}")
        if self.window < 0 or self.keep_first < 0 or self.softcap < 0:
            raise ValueError(f"attention: window, keep_first and softcap must not be negative: {self}")
        if self.pool < 0 or (self.pool and (not self.window or self.keep_first or self.kv_from is not None)):
            raise ValueError(f"attention: pooled blocks lie behind a window: {self}")
        if self.rot is not None and self.rot.dims > self.dim:
            raise ValueError(f"attention: rot dims {self.rot.dims} exceed a head's {self.dim}")
        if self.qk_norm not in (None, HEAD, WHOLE) or self.temp_every < 1 or (self.distance_bias and not self.sigmoid) \
                or (self.head_gate and self.elem_gate) or (self.sink and self.sigmoid) \
                or (self.prepared and self.kv_from is not None):
            raise ValueError(f"attention: these do not go together: {self}")
        if self.tied_values and (self.dim != self.vdim or self.kv_from is not None):
            raise ValueError(f"attention: values that are the keys have their size: {self}")

    @property
    def prepared(self) -> bool:
        """Queries and keys change between projection and score."""
        return self.qk_norm is not None or self.rot is not None or self.tied_values

    def temperature(self, p: int) -> float:
        return 1.0 + self.temp_coef * math.log((p + 1) // self.temp_every + 1)

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
        """Values per token in this layer's cache (0: it reads another layer's), its share of a pooled
        block's among them."""
        if self.kv_from is not None:
            return 0
        n = self.kv_heads * (self.dkp + self.dvp)
        return n + (-(-n // self.pool) if self.pool else 0)

    @property
    def state_bytes(self) -> int:
        return 0

    @property
    def scratch_width(self) -> int:
        own = self.kv_heads * (self.dkp + self.dvp) if self.kv_from is None else 0
        gate = self.heads * self.dvp if self.elem_gate else pad_to(self.heads, 16)
        return self.heads * (self.dkp + self.dvp) + own + gate

    def part_bytes(self, items: int, elem_bytes: int) -> int:
        return items * self.heads * (self.dvp + 2) * 4

    def params(self, width: int) -> int:
        n = self.heads * self.dim * (width + self.bias) + self.heads * self.vdim * width + width * self.out_bias
        if self.kv_from is None:
            n += self.kv_heads * (self.dim + (0 if self.tied_values else self.vdim)) * (width + self.bias)
        n += {None: 0, HEAD: 2 * self.dim, WHOLE: (self.heads + self.kv_heads) * self.dim}[self.qk_norm]
        n += self.heads * (2 * self.distance_bias + self.sigmoid) + self.heads * self.vdim * width * self.elem_gate
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
        return pad_state(self.dim, self.vdim)

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


def pad_state(dim: int, vdim: int) -> tuple:
    """(key channels, value channels) of a head's state as stored: a kernel's size, or as they are beyond."""
    if max(dim, vdim) > 128:
        return dim, vdim
    return tuple(next(k for k in (32, 64, 128) if n <= k) for n in (dim, vdim))


@dataclass(frozen=True)
class RetentionSpec:
    """Linear attention with a fixed decay per head: per head a state S [dim, vdim],

        S <- decay S + k v^T;  o = S^T q

    q and k are rotated, k times ``k_scale``; o is RMS-normed over vdim and multiplied by silu of a projected
    gate."""
    heads: int
    dim: int
    vdim: int
    decay: tuple
    k_scale: float
    rot: Optional[RotarySpec] = None

    cache_width = 0

    def __post_init__(self):
        if min(self.heads, self.dim, self.vdim) < 1 or len(self.decay) != self.heads:
            raise ValueError(f"retention: bad sizes: {self}")
        if not all(0 < d <= 1 for d in self.decay):
            raise ValueError(f"retention: decays lie in (0, 1]: {self}")
        if self.rot is not None and self.rot.dims > self.dim:
            raise ValueError(f"retention: rot dims {self.rot.dims} exceed a head's {self.dim}")

    @property
    def state_dims(self) -> tuple:
        return pad_state(self.dim, self.vdim)

    @property
    def state_bytes(self) -> int:
        dk, dv = self.state_dims
        return 4 * self.heads * dk * dv

    @property
    def scratch_width(self) -> int:
        return self.heads * (2 * self.dim + 3 * self.vdim)

    def part_bytes(self, items: int, elem_bytes: int) -> int:
        return 0

    def params(self, width: int) -> int:
        return self.heads * (2 * self.dim + 3 * self.vdim) * width


@dataclass(frozen=True)
class MlstmSpec:
    """Matrix memory (mLSTM): per head a state S [dim, vdim], n [dim] and a running maximum m, all from zero. With
    log gates i = gate_cap tanh(. / gate_cap) and f = log sigmoid(gate_cap tanh(. / gate_cap)) of projected numbers,

        m' = max(f + m, i);  S <- exp(f + m - m') S + exp(i - m') k v^T;  n <- the same with k alone;  m <- m'
        o = S^T q / (max(|n . q|, exp(-m)) + 1e-6)

    q times ``q_scale``; o is RMS-normed per head, weighted and multiplied by the sigmoid of a projected gate."""
    heads: int
    dim: int
    vdim: int
    gate_cap: float
    q_scale: float

    cache_width = 0

    def __post_init__(self):
        if min(self.heads, self.dim, self.vdim) < 1 or not self.gate_cap > 0:
            raise ValueError(f"matrix memory: bad values: {self}")

    @property
    def state_dims(self) -> tuple:
        return pad_state(self.dim, self.vdim)

    @property
    def copies(self) -> int:
        """Times n and m are stored: once per slice of the value channels that a workgroup of its own advances
        (csrc/kernels/mlstm.h)."""
        return 2 if self.state_dims[1] == 128 and self.state_dims[0] <= 128 else 1

    @property
    def state_bytes(self) -> int:
        dk, dv = self.state_dims
        return 4 * self.heads * (dk * dv + self.copies * (dk + 1))

    @property
    def scratch_width(self) -> int:
        dk, dv = self.state_dims
        return self.heads * (2 * dk + 3 * dv) + 4 * pad_to(self.heads, 16) + 256

    def part_bytes(self, items: int, elem_bytes: int) -> int:
        return 0

    def params(self, width: int) -> int:
        H = self.heads
        return H * (2 * self.dim + 3 * self.vdim) * width + 2 * H * (width + 1) + H * self.vdim


@dataclass(frozen=True)
class PairSpec:
    """Attention and a recurrent mixer side by side on one input: left_scale * left + right_scale * right."""
    left: AttentionSpec
    right: RetentionSpec
    left_scale: float
    right_scale: float

    @property
    def heads(self) -> int:
        return self.left.heads

    @property
    def cache_width(self) -> int:
        return self.left.cache_width

    @property
    def state_bytes(self) -> int:
        return self.right.state_bytes

    @property
    def scratch_width(self) -> int:
        return self.left.scratch_width + self.right.scratch_width

    def part_bytes(self, items: int, elem_bytes: int) -> int:
        return self.left.part_bytes(items, elem_bytes)

    def params(self, width: int) -> int:
        return self.left.params(width) + self.right.params(width)


def leaves(mixer) -> list:
    """The mixers that a mixer is made of."""
    return [mixer.left, mixer.right] if isinstance(mixer, PairSpec) else [mixer]


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


SILU_GLU, RELU2 = "silu_glu", "relu2"  # an expert: W_down (silu(W_gate h) * W_up h) / W_down relu(W_up h)^2


@dataclass(frozen=True)
class MoeSpec:
    """``experts`` small feed-forwards (``act``) of which a token uses ``top``: those with the largest router
    logits, weighted by the softmax over these; or with ``sigmoid`` those with the largest sigmoid of the
    logit plus a ``correction`` per expert, among the ``keep`` of ``groups`` equal groups of neighbours whose
    two best choices sum highest, weighted by the sigmoids over their sum, times ``scale``. ``shared_ff``: one
    more expert of this size that every token uses, with ``shared_gate`` times the sigmoid of one projected number.
    ``bias``: the router has one."""
    experts: int
    top: int
    ff: int
    act: str = SILU_GLU
    sigmoid: bool = False
    correction: bool = False
    groups: int = 1
    keep: int = 1
    scale: float = 1.0
    shared_ff: int = 0
    shared_gate: bool = False
    bias: bool = False

    def __post_init__(self):
        if min(self.experts, self.top, self.ff) < 1 or self.top > self.experts or self.shared_ff < 0:
            raise ValueError(f"experts: bad sizes: {self}")
        if self.act not in (SILU_GLU, RELU2) or (self.shared_gate and not self.shared_ff):
            raise ValueError(f"experts: unknown kind: {self}")
        if not 1 <= self.keep <= self.groups or self.experts % self.groups \
                or self.top > self.keep * (self.experts // self.groups):
            raise ValueError(f"experts: bad groups: {self}")
        if not self.sigmoid and (self.groups > 1 or self.correction or self.scale != 1.0):
            raise ValueError(f"experts: groups, corrections and scales go with sigmoid scores: {self}")

    @property
    def mats(self) -> int:
        """Matrices of an expert."""
        return 3 if self.act == SILU_GLU else 2

    def scratch_width(self, width: int) -> int:
        return 2 * pad_to(self.experts + self.shared_gate, 128) + self.top * (pad_to(self.ff, 128) + 2 * pad_to(width, 128) + 8) \
            + pad_to(self.shared_ff, 128) + (2 * pad_to(width, 128) if self.shared_ff else 0)

    def params(self, width: int) -> int:
        return (self.experts * (self.mats * self.ff + 1) + self.mats * self.shared_ff + self.shared_gate) * width \
            + self.experts * self.bias

    def active_params(self, width: int) -> int:
        """Weights one token uses."""
        return (self.mats * (self.ff * self.top + self.shared_ff) + self.experts + self.shared_gate) * width


# How a layer's sublayers meet the residual stream
POST_NORM = "post_norm"  # each sublayer reads the stream; its result is normed, scaled per element and added
PARALLEL = "parallel"    # both read one norm of the stream; each result is added through a sigmoid gate per element
SANDWICH = "sandwich"    # each sublayer reads a norm of the stream; its result is normed again and added
HYPER = "hyper"          # several streams: each sublayer reads a norm of a weighted sum of them; a matrix mixes them anew


@dataclass(frozen=True)
class LayerSpec:
    mixer: Any  # LatentSpec | AttentionSpec | DeltaSpec | RetentionSpec | MlstmSpec | PairSpec
    mlp: Any    # GluSpec | DenseSpec | MoeSpec | None
    owner: int  # number, in the tensors' names, of the layer whose tensors this one uses
    block: str = POST_NORM
    enters: Optional[int] = None  # a pass of this number begins here: x <- W_in [x; embedding output] + step


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
    streams: int = 1           # copies of the residual stream; the head reads their sum
    logit_scale: float = 1.0
    logit_softcap: float = 0.0  # logits become softcap tanh(logits / softcap) (0: as they are)
    raw: Optional[dict] = None  # the config.json it was read from

    is_gpt2 = False

    # ------------------------------------------------------------------ framework view
    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @property
    def stream_width(self) -> int:
        """Values of one row between layers and stages."""
        return self.streams * self.hidden_size

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
        elif s.block == HYPER:
            coef = self.streams * (self.streams + 2)
            n, extra = s.mixer.params(W) + W + coef, W + coef
        elif s.enters is not None:
            n, extra = s.mixer.params(W) + 2 * W + 2 * W * W + W, 2 * W
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
        runs on the stage that holds them, one that reads the embedding output on the first."""
        tied = set()
        for i, s in enumerate(self.layers):
            if s.enters is not None:
                tied.update(range(1, i + 1))
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
        n = rows * (self.stream_width * 4 + W * (4 + elem_bytes) + 12)
        inter = part = 0
        for l in self.layers:
            gates = 2 * pad_to(self.hidden_size, 16) if l.block == PARALLEL else 0
            gates += 4 * W if l.enters is not None else 0
            inter = max(inter, l.mixer.scratch_width + gates
                        + (l.mlp.scratch_width(self.hidden_size) if l.mlp is not None else 0) + 5 * 128)
            part = max(part, l.mixer.part_bytes(1024, elem_bytes))
        return n + rows * inter * elem_bytes + part + (1 << 26) + 2 * 256 * 256 * 256 * 4

    def stream_bytes(self) -> int:
        """Bytes of one row of the residual stream between pipeline stages (fp32)."""
        return 4 * self.stream_width

    def to_dict(self) -> dict:
        if self.raw is None:
            raise ValueError("this configuration was not read from a config.json")
        return self.raw


__all__ = ["StackConfig", "LayerSpec", "LatentSpec", "AttentionSpec", "DeltaSpec", "RetentionSpec", "MlstmSpec", "PairSpec", "RotarySpec",
           "GluSpec", "DenseSpec", "MoeSpec", "POST_NORM", "PARALLEL", "SANDWICH", "HYPER", "HEAD", "WHOLE", "SILU_GLU", "RELU2",
           "leaves", "pad_to", "pad_part"]
