"""Projections of a stack engine, and the kernels of its fp32 residual stream (csrc/kernels/stream_ops.hip,
linear_f32.hip): what every mixer and feed-forward of a stack shares.

The conventions of :mod:`.hip` hold: shapes are checked on the host, launches go to torch's current
stream, nothing falls back to another implementation."""
from __future__ import annotations

import ctypes
from typing import Optional

import torch

from . import hip
from .hip import _check, _p, _req, _stream, lib
from .packing import fuse_gate_up, pack_b


def is_f32(dt) -> int:
    _req(dt in (torch.float32, torch.bfloat16), f"unsupported compute type {dt}")
    return int(dt == torch.float32)


# ------------------------------------------------------------------------------ projections
def pad2(w: torch.Tensor, n: int, k: int) -> torch.Tensor:
    """[N, K] -> [n, k], zeros behind."""
    out = torch.zeros((n, k), dtype=w.dtype, device=w.device)
    out[:w.shape[0], :w.shape[1]] = w
    return out


class Linear:
    """One projection of a stack engine in the engine's type: N and K padded to whole 128-wide
    blocks with zeros, so that every kernel configuration takes it; bf16 weights packed for
    the MFMA kernels, fp32 ones row-major."""

    def __init__(self, w: torch.Tensor, k: int = 0):
        N, K = w.shape
        self.n, self.k = -(-N // 128) * 128, k or -(-K // 128) * 128
        wp = w if w.shape == (self.n, self.k) else pad2(w, self.n, self.k)
        self.f32 = is_f32(w.dtype)
        self.w = wp.contiguous() if self.f32 else pack_b(wp).contiguous()

    @staticmethod
    def glu(gate: torch.Tensor, up: torch.Tensor) -> "Linear":
        """Gate and up projection, interleaved for the gated epilogue; ff padded to 128."""
        ff, K = gate.shape
        n = -(-ff // 128) * 128
        return Linear(fuse_gate_up(pad2(gate, n, K), pad2(up, n, K)))

    @staticmethod
    def glu_bias(gate: torch.Tensor, up: torch.Tensor) -> torch.Tensor:
        """Biases [ff] of both, in the order of :meth:`glu`'s columns."""
        n = -(-gate.numel() // 128) * 128
        return fuse_gate_up(pad2(gate[:, None], n, 1), pad2(up[:, None], n, 1)).reshape(-1).contiguous()

    def tensors(self) -> list:
        return [self.w]

    def __call__(self, x: torch.Tensor, rows: int, out: Optional[torch.Tensor], ws=None, sk_ws=None, glu=None, keys=None,
                 bias=None, col_offset: int = 0, out32: Optional[torch.Tensor] = None, col32: int = 0,
                 act_from: Optional[int] = None, act: int = hip.ACT_GELU, gate: Optional[torch.Tensor] = None,
                 cols: int = 0) -> None:
        """out[:rows] = x[:rows] . W^T (``out`` in the engine's type or fp32), or with ``glu`` (a GluSpec) the
        gated unit of the interleaved halves; ``keys``: argmax keys instead of an output.
        ``out32`` beside ``out``: columns from ``col32`` on go there, in fp32; ``act_from``: the activation ``act``
        on the other columns from there on. ``out32`` alone with ``gate``: out32[:, :cols] += sigmoid(gate) * result."""
        _req(x.dim() == 2 and x.shape[0] >= rows and x.shape[1] >= self.k and x.stride(1) == 1, "linear: input shape")
        kw = {}
        if keys is None:
            n_out = self.n // 2 if glu is not None else (self.n if out32 is None else col32)
            if out is None:
                _req(out32 is not None and gate is not None and gate.dtype == x.dtype and gate.shape[0] >= rows
                     and 0 < cols <= min(out32.shape[1], self.n), "linear: gated accumulation")
                kw.update(out32=out32, ldo=out32.stride(0), gate=gate, cols=cols)
            else:
                _req(out.shape[0] >= rows and out.shape[1] >= n_out and out.stride(1) == 1, "linear: output shape")
                kw["ldo"] = out.stride(0)
                if out32 is not None:
                    _req(out.dtype == x.dtype, "linear: two outputs")
                    kw.update(out=out, out32=out32, col32=col32, ldo32=out32.stride(0))
                elif out.dtype == torch.float32 and not self.f32:
                    kw["out32"] = out
                else:
                    kw["out32" if glu is not None and self.f32 else "out"] = out
            if out32 is not None:
                _req(out32.dtype == torch.float32 and out32.shape[0] >= rows and out32.stride(1) == 1
                     and (gate is not None or out32.shape[1] >= self.n - col32), "linear: fp32 output shape")
        if act_from is not None:
            kw.update(act=act, act_from=act_from)
        if glu is not None:
            _req(bias is None or glu.gelu, "linear: biases of a gated product go with gelu")
            kw.update(glu_alpha=glu.alpha, glu_limit=glu.limit, glu_shift=glu.shift)
        _req(bias is None or bias.numel() >= self.n, "linear: bias")
        epi = (hip.EPI_GEGLU if glu.gelu else hip.EPI_SWIGLU) if glu is not None else (hip.EPI_STORE if keys is None else hip.EPI_ARGMAX)
        ep = hip.make_epi(keys=keys, bias=bias, col_offset=col_offset, **kw)
        if self.f32:
            _req(x.dtype == torch.float32 and x.is_cuda and keys is None, "linear: fp32 cuda input")
            _check(lib().lsa_linear_f32(_p(x), x.stride(0), _p(self.w), rows, self.n, self.k, epi, ctypes.byref(ep),
                                        _stream()), "lsa_linear_f32")
        elif rows <= 128:
            hip.gemv(x, self.w, rows, self.n, self.k, epi, ep, ws=ws)
        else:
            hip.gemm_sk(x, self.w, rows, self.n, self.k, epi, ep, ws=sk_ws)


# ------------------------------------------------------------------------------ fp32 stream
def stream_embed(ids, table, scale: float, x, xc, rows: int, copies: int = 1) -> None:
    """x = table[ids] * scale, ``copies`` of it side by side; ``xc`` (or None): one in the projections' type."""
    W = x.shape[1] // copies
    _req(ids.dtype == torch.int32 and ids.is_cuda and ids.numel() >= rows, "stream_embed: int32 ids")
    _req(x.dtype == torch.float32 and x.shape[0] >= rows and x.shape[1] == W * copies and table.shape[1] >= W, "stream_embed: shapes")
    _req(xc is None or (table.dtype == xc.dtype and xc.shape[1] >= W and xc.shape[0] >= rows), "stream_embed: copy")
    _check(lib().lsa_stream_embed(is_f32(table.dtype), _p(ids), rows, _p(table), table.stride(0), float(scale), W, copies, _p(x),
                                  x.stride(0), _p(xc), 0 if xc is None else xc.stride(0), _stream()), "lsa_stream_embed")


def cast_rows(x, xc, rows: int, x2=None) -> None:
    """xc = x in the projections' type; ``x2`` (fp32): a copy as it is."""
    _req(x.dtype == torch.float32 and x.stride(1) == 1 and xc.shape[1] >= x.shape[1]
         and min(x.shape[0], xc.shape[0]) >= rows, "cast_rows: shapes")
    _req(x2 is None or (x2.dtype == torch.float32 and x2.shape[0] >= rows and x2.shape[1] >= x.shape[1]), "cast_rows: x2")
    _check(lib().lsa_cast_rows(is_f32(xc.dtype), _p(x), x.stride(0), rows, x.shape[1], _p(xc), xc.stride(0), _p(x2),
                               0 if x2 is None else x2.stride(0), _stream()), "lsa_cast_rows")


def stream_add_norm(y, gain, eps: float, x, xc, rows: int) -> None:
    """x += rms(y) * gain; xc = x in the projections' type."""
    W = gain.numel()
    _req(all(t.dtype == torch.float32 for t in (y, gain, x)) and y.shape[1] >= W and x.shape[1] >= W and xc.shape[1] >= W
         and min(t.shape[0] for t in (y, x, xc)) >= rows, "stream_add_norm: shapes")
    _check(lib().lsa_stream_add_norm(is_f32(xc.dtype), _p(y), y.stride(0), _p(gain), float(eps), rows, W, _p(x),
                                     x.stride(0), _p(xc), xc.stride(0), _stream()), "lsa_stream_add_norm")


def stream_norm(x, gain, eps: float, out, rows: int) -> None:
    W = gain.numel()
    _req(x.dtype == torch.float32 and gain.dtype == torch.float32 and x.shape[1] >= W and out.shape[1] >= W
         and min(x.shape[0], out.shape[0]) >= rows, "stream_norm: shapes")
    _check(lib().lsa_stream_norm(is_f32(out.dtype), _p(x), x.stride(0), _p(gain), float(eps), rows, W, _p(out),
                                 out.stride(0), _stream()), "lsa_stream_norm")


class JoinArgs(ctypes.Structure):
    _fields_ = ([(n, ctypes.c_void_p) for n in ("y1", "g1", "g2", "y2", "ye", "weight", "place", "gain")]
                + [(n, ctypes.c_int) for n in ("ldy1", "ldg1", "ldg2", "ldy2", "ldye", "top")] + [("eps", ctypes.c_float)])


def stream_join(x, rows: int, first=None, second=None, experts=None, gate2=None, gain=None, eps: float = 0.0,
                out=None) -> None:
    """x += sigmoid(gate) * y for ``first`` = (y fp32, gate), and with ``gate2`` for ``second`` (fp32 y) or
    ``experts`` = (results of the sorted pairs, weights, places, top: a row's weighted sum). With ``gain`` then
    out = rms(x) * gain in the projections' type."""
    W, dt = x.shape[1], None
    y1, g1 = first if first is not None else (None, None)
    ye, weight, place, top = experts if experts is not None else (None, None, None, 0)
    _req(x.dtype == torch.float32 and x.stride(1) == 1 and x.shape[0] >= rows, "join: stream")
    _req((second is None or experts is None) and (gate2 is not None) == (second is not None or experts is not None),
         "join: one second result and its gate")
    for t in (y1, second):
        _req(t is None or (t.dtype == torch.float32 and t.shape[0] >= rows and t.shape[1] >= W and t.stride(1) == 1),
             "join: fp32 result")
    for t in (g1, gate2, ye, out):
        _req(t is None or (t.stride(1) == 1 and t.shape[1] >= W and t.shape[0] >= rows and dt in (None, t.dtype)),
             "join: types and shapes")
        dt = dt if t is None else t.dtype
    _req(experts is None or (ye.shape[0] >= rows * top and min(weight.numel(), place.numel()) >= rows * top
                             and weight.dtype == torch.float32 and place.dtype == torch.int32), "join: experts")
    _req(gain is None or (gain.dtype == torch.float32 and gain.numel() == W and out is not None), "join: norm")
    if dt is None:
        return

    def ld(t):
        return 0 if t is None else t.stride(0)
    a = JoinArgs(_p(y1), _p(g1), _p(gate2), _p(second), _p(ye), _p(weight), _p(place), _p(gain), ld(y1), ld(g1), ld(gate2),
                 ld(second), ld(ye), top, float(eps))
    _check(lib().lsa_stream_join(is_f32(dt), ctypes.byref(a), rows, W, _p(x), x.stride(0), _p(out), ld(out), _stream()),
           "lsa_stream_join")


class RenormArgs(ctypes.Structure):
    _fields_ = ([(n, ctypes.c_void_p) for n in ("y", "ye", "weight", "place", "post", "gain")]
                + [(n, ctypes.c_int) for n in ("ldy", "ldye", "top", "add")] + [("eps", ctypes.c_float)])


def stream_renorm(x, rows: int, y=None, experts=None, post=None, gain=None, eps: float = 0.0, out=None,
                  add: bool = True) -> None:
    """x += rms(v) * post (``post`` None: v; not ``add``: x becomes that), v = ``y`` (fp32) plus, with ``experts`` =
    (results of the sorted pairs, weights, places, top), a row's weighted sum; then out = rms(x) * gain (``gain``
    None: x) in the projections' type."""
    W = x.shape[1]
    ye, weight, place, top = experts if experts is not None else (None, None, None, 0)
    _req(x.dtype == torch.float32 and x.stride(1) == 1 and x.shape[0] >= rows, "renorm: stream")
    _req(y is not None or ye is not None, "renorm: nothing joins")
    _req(y is None or (y.dtype == torch.float32 and y.shape[0] >= rows and y.shape[1] >= W and y.stride(1) == 1), "renorm: y")
    _req(ye is None or (ye.stride(1) == 1 and ye.shape[1] >= W and ye.shape[0] >= rows * top
                        and min(weight.numel(), place.numel()) >= rows * top and weight.dtype == torch.float32
                        and place.dtype == torch.int32), "renorm: experts")
    _req(out is None or (out.stride(1) == 1 and out.shape[1] >= W and out.shape[0] >= rows
                         and (ye is None or ye.dtype == out.dtype)), "renorm: copy")
    for g in (post, gain):
        _req(g is None or (g.dtype == torch.float32 and g.numel() == W), "renorm: norm weights")
    _req(gain is None or out is not None, "renorm: a norm needs a place")

    def ld(t):
        return 0 if t is None else t.stride(0)
    a = RenormArgs(_p(y), _p(ye), _p(weight), _p(place), _p(post), _p(gain), ld(y), ld(ye), top, int(add), float(eps))
    dt = ye.dtype if ye is not None else out.dtype if out is not None else torch.float32
    _check(lib().lsa_stream_renorm(is_f32(dt), ctypes.byref(a), rows, W, _p(x), x.stride(0), _p(out), ld(out), _stream()),
           "lsa_stream_renorm")


class MixArgs(ctypes.Structure):
    _fields_ = ([(n, ctypes.c_void_p) for n in ("coef", "y", "ygate", "ye", "weight", "place", "read", "gain")]
                + [(n, ctypes.c_int) for n in ("streams", "ldy", "ldyg", "ldye", "top")] + [("eps", ctypes.c_float)])


MAX_STREAMS = 16  # of stream_mix (MAXS in csrc/kernels/stream_mix.hip)


def stream_mix(x, rows: int, streams: int, coef=None, y=None, ygate=None, experts=None, read=None, eps: float = 0.0,
               out=None) -> None:
    """Rows of ``streams`` streams x_s side by side. With ``coef`` = [out | mix] (fp32): x_t <- sum_s mix[s, t] x_s +
    out[t] v, v = ``y`` (fp32), times the sigmoid of ``ygate`` [rows, 1..] (fp32) where given, plus with ``experts`` =
    (results of the sorted pairs, weights, places, top) a row's weighted sum. With ``read`` (its ``weights`` and
    ``gain``, fp32) then out = rms(sum_s weights[s] x_s) * gain in the projections' type."""
    _req(1 <= streams <= MAX_STREAMS and x.shape[1] % streams == 0, f"mix: 1 to {MAX_STREAMS} streams")
    W = x.shape[1] // streams
    ye, weight, place, top = experts if experts is not None else (None, None, None, 0)
    _req(x.dtype == torch.float32 and x.stride(1) == 1 and x.shape[0] >= rows, "mix: streams")
    _req((coef is None) == (y is None and ye is None) and (coef is not None or read is not None), "mix: nothing to do")
    _req(coef is None or (coef.dtype == torch.float32 and coef.numel() == streams * (streams + 1) and coef.is_contiguous()),
         "mix: coefficients")
    _req(y is None or (y.dtype == torch.float32 and y.shape[0] >= rows and y.shape[1] >= W and y.stride(1) == 1), "mix: y")
    _req(ygate is None or (y is not None and ygate.dtype == torch.float32 and ygate.shape[0] >= rows), "mix: gate")
    _req(ye is None or (ye.stride(1) == 1 and ye.shape[1] >= W and ye.shape[0] >= rows * top
                        and min(weight.numel(), place.numel()) >= rows * top and weight.dtype == torch.float32
                        and place.dtype == torch.int32), "mix: experts")
    wts, gain = (read.weights, read.gain) if read is not None else (None, None)
    if read is None:
        out = None
    else:
        _req(wts.dtype == gain.dtype == torch.float32 and wts.numel() == streams and gain.numel() == W
             and wts.is_contiguous() and gain.is_contiguous(), "mix: read")
        _req(out is not None and out.stride(1) == 1 and out.shape[1] >= W and out.shape[0] >= rows
             and (ye is None or ye.dtype == out.dtype), "mix: copy")

    def ld(t):
        return 0 if t is None else t.stride(0)
    a = MixArgs(_p(coef), _p(y), _p(ygate), _p(ye), _p(weight), _p(place), _p(wts), _p(gain), streams, ld(y), ld(ygate), ld(ye),
                top, float(eps))
    dt = ye.dtype if ye is not None else out.dtype if out is not None else torch.float32
    _check(lib().lsa_stream_mix(is_f32(dt), ctypes.byref(a), rows, W, _p(x), x.stride(0), _p(out), ld(out), _stream()),
           "lsa_stream_mix")


def softcap_rows(lg, rows: int, n: int, cap: float) -> None:
    """lg[:rows, :n] becomes cap * tanh(lg / cap)."""
    _req(lg.dtype == torch.float32 and lg.stride(1) == 1 and lg.shape[0] >= rows and lg.shape[1] >= n and cap > 0, "softcap_rows: shapes")
    _check(lib().lsa_softcap_rows(_p(lg), lg.stride(0), rows, n, float(cap), _stream()), "lsa_softcap_rows")


def logits_argmax(lg, rows: int, vocab: int, keys, offset: int = 0) -> None:
    _req(lg.dtype == torch.float32 and lg.shape[0] >= rows and lg.shape[1] >= vocab and keys.dtype == torch.int64
         and keys.numel() >= rows, "logits_argmax: shapes")
    _check(lib().lsa_logits_argmax(_p(lg), lg.stride(0), rows, vocab, offset, _p(keys), _stream()), "lsa_logits_argmax")


def declare(L: ctypes.CDLL) -> None:
    """Signatures of these entry points (called by hip.load_library)."""
    vp, i, f = ctypes.c_void_p, ctypes.c_int, ctypes.c_float
    hip.set_signatures(L, {
        "lsa_stream_embed": [i, vp, i, vp, i, f, i, i, vp, i, vp, i, vp],
        "lsa_stream_mix": [i, ctypes.POINTER(MixArgs), i, i, vp, i, vp, i, vp],
        "lsa_softcap_rows": [vp, i, i, i, f, vp],
        "lsa_cast_rows": [i, vp, i, i, i, vp, i, vp, i, vp],
        "lsa_stream_add_norm": [i, vp, i, vp, f, i, i, vp, i, vp, i, vp],
        "lsa_stream_norm": [i, vp, i, vp, f, i, i, vp, i, vp],
        "lsa_stream_join": [i, ctypes.POINTER(JoinArgs), i, i, vp, i, vp, i, vp],
        "lsa_stream_renorm": [i, ctypes.POINTER(RenormArgs), i, i, vp, i, vp, i, vp],
        "lsa_logits_argmax": [vp, i, i, i, i, vp, vp],
        "lsa_linear_f32": [vp, i, vp, i, i, i, i, ctypes.POINTER(hip.EpiArgs), vp],
    })
