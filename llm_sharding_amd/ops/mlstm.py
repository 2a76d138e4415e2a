"""Bindings of the matrix memory kernels (csrc/kernels/mlstm*.hip).

The conventions of :mod:`.hip` hold: shapes are checked on the host, launches go to torch's current
stream, nothing falls back to another implementation."""
from __future__ import annotations

import ctypes

import torch

from . import hip
from .delta import check_runs  # noqa: F401  (one run per slot and step, as there)
from .hip import _check, _p, _req, _stream, lib
from .retention import segments  # noqa: F401  (of 64-row chunks, as there)
from .stream import is_f32


class MlArgs(ctypes.Structure):
    _fields_ = ([(n, ctypes.c_void_p) for n in ("inp", "in32", "S", "n", "m", "norm", "runs", "slot", "pos", "table", "out")]
                + [(n, ctypes.c_int) for n in ("ldi", "ldi32", "ldo", "oq", "ok", "ov", "og", "oi", "of", "heads", "dim", "vdim",
                                               "dk", "dv", "copies", "max_pages", "n_pages")]
                + [(n, ctypes.c_float) for n in ("cap", "q_scale", "eps")])


def make_args(s, norm, state: tuple, inp, in32, cols: tuple, gates: tuple, out, eps: float, table, n_pages: int, slot=None,
              pos=None, runs=None) -> MlArgs:
    """``norm`` fp32 [heads dv]; ``state``: S, n and m, fp32 [slots, heads, ...]; ``cols``: first columns of q, k, v and
    gate in ``inp``, ``gates``: of the input and forget gates in ``in32``; ``runs`` int32 [n, 4] (row0, rows, slot, pos0),
    checked by :func:`check_runs`, or ``slot`` / ``pos`` int32 [rows]."""
    S, n, m = state
    dk, dv = s.state_dims
    _req(all(t.dtype == torch.float32 and t.is_contiguous() for t in (S, n, m, norm)) and norm.numel() == s.heads * dv
         and tuple(S.shape[1:]) == (s.heads, dk, dv) and tuple(n.shape) == S.shape[:2] + (s.copies, dk)
         and tuple(m.shape) == n.shape[:3], "mlstm: state")
    kc, vc = s.heads * dk, s.heads * dv
    _req(inp.dtype == out.dtype and inp.stride(1) == out.stride(1) == 1 and out.shape[0] >= inp.shape[0]
         and out.shape[1] >= vc and inp.shape[1] >= max(cols[0] + kc, cols[1] + kc, cols[2] + vc, cols[3] + vc),
         "mlstm: inputs")
    _req(in32.dtype == torch.float32 and in32.stride(1) == 1 and in32.shape[0] >= inp.shape[0]
         and in32.shape[1] >= max(gates) + s.heads, "mlstm: gates")
    _req((runs is None) != (slot is None), "mlstm: runs or rows")
    _req(table.dtype == torch.int32 and table.shape[0] <= S.shape[0], "mlstm: page table")
    for t in (runs, slot, pos):
        _req(t is None or (t.dtype == torch.int32 and t.is_contiguous()), "mlstm: int32 rows")
    return MlArgs(_p(inp), _p(in32), _p(S), _p(n), _p(m), _p(norm), _p(runs), _p(slot), _p(pos), _p(table), _p(out),
                  inp.stride(0), in32.stride(0), out.stride(0), *cols, *gates, s.heads, s.dim, s.vdim, dk, dv, s.copies,
                  table.shape[1], n_pages, float(s.gate_cap), float(s.q_scale), float(eps))


def chunk_size(s) -> bool:
    """The chunked kernels take this size."""
    return max(s.state_dims) <= 128


def chunked(a: MlArgs, s, items, longest: int, several: bool, gates, rows: int, parts: tuple, o32) -> None:
    """The segments of checked runs, bf16: ``items`` (device), ``gates`` fp32 [3 heads rows]; ``parts`` (with several
    segments per run): fp32 workspaces of S, n and m by entry; ``o32`` fp32 [rows, heads dv]."""
    _req(o32.dtype == torch.float32 and o32.stride(1) == 1 and o32.shape[0] >= rows and o32.shape[1] >= s.heads * s.state_dims[1],
         "mlstm: read-outs")
    _req(items.dtype == torch.int32 and items.is_contiguous() and items.shape[1] == 8, "mlstm: segments")
    _req(gates.dtype == torch.float32 and gates.is_contiguous() and gates.numel() >= 3 * s.heads * rows, "mlstm: gates")
    _req(not several or all(t.dtype == torch.float32 and t.is_contiguous() for t in parts), "mlstm: workspace")
    _check(lib().lsa_ml_chunked(ctypes.byref(a), _p(items), items.shape[0], longest, int(several), _p(gates), rows,
                                *(_p(t) for t in (parts if several else (None,) * 3)), _p(o32), o32.stride(0), _stream()),
           "lsa_ml_chunked")


def steps(a: MlArgs, dtype, n: int) -> None:
    """n runs (or rows), step by step."""
    _check(lib().lsa_ml_steps(is_f32(dtype), ctypes.byref(a), n, _stream()), "lsa_ml_steps")


def declare(L: ctypes.CDLL) -> None:
    """Signatures of these entry points (called by hip.load_library)."""
    vp, i = ctypes.c_void_p, ctypes.c_int
    ma = ctypes.POINTER(MlArgs)
    hip.set_signatures(L, {"lsa_ml_steps": [i, ma, i, vp],
                           "lsa_ml_chunked": [ma, vp, i, i, i, vp, i, vp, vp, vp, vp, i, vp]})
