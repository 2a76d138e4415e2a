"""Bindings of the gated delta rule kernels (csrc/kernels/delta*.hip).

The conventions of :mod:`.hip` hold: shapes are checked on the host, launches go to torch's current
stream, nothing falls back to another implementation."""
from __future__ import annotations

import ctypes

import torch

from . import hip
from .hip import _check, _p, _req, _stream, lib
from .stream import is_f32


class DeltaArgs(ctypes.Structure):
    _fields_ = ([(n, ctypes.c_void_p) for n in ("inp", "in32", "z", "gate", "conv", "decay", "dt_bias", "norm", "state",
                                                "ring", "runs", "slot", "pos", "table", "out")]
                + [(n, ctypes.c_int) for n in ("ldi", "ld32", "ldz", "ldg", "ldo", "oq", "ok", "ov", "ob", "heads",
                                               "kv_heads", "dim", "vdim", "taps", "dk", "dv", "max_pages", "n_pages")]
                + [("q_scale", ctypes.c_float), ("unit_eps", ctypes.c_float), ("eps", ctypes.c_float)])


def state_shapes(s, slots: int) -> tuple:
    """(state, ring of convolution inputs) of one layer, fp32."""
    return (slots, s.heads) + s.state_dims, (slots, s.taps, s.channels)


def make_args(s, w: dict, state: tuple, inp, cols: tuple, in32, ob: int, z, gate, out, eps: float, table, n_pages: int,
              slot=None, pos=None, runs=None) -> DeltaArgs:
    """``w``: conv [channels, taps], decay [heads], dt_bias [heads dim], norm [vdim], fp32; ``cols``: first columns
    of q, k and v in ``inp``; ``ob``: of the step sizes in ``in32``; ``runs`` int32 [n, 4] (row0, rows, slot,
    pos0), checked by :func:`check_runs`, or ``slot`` / ``pos`` int32 [rows]."""
    S, ring = state
    rows = inp.shape[0]
    _req(all(t.dtype == torch.float32 and t.is_contiguous() for t in (S, ring, *w.values())), "delta: fp32 state, weights")
    _req(tuple(S.shape[1:]) == (s.heads,) + s.state_dims and tuple(ring.shape) == (S.shape[0], s.taps, s.channels),
         "delta: state shapes")
    _req(w["conv"].shape == (s.channels, s.taps) and w["decay"].numel() == s.heads and w["norm"].numel() == s.vdim
         and w["dt_bias"].numel() == s.heads * s.dim, "delta: weights")
    _req(in32.dtype == z.dtype == torch.float32 and gate.dtype == inp.dtype == out.dtype
         and all(t.stride(1) == 1 and t.shape[0] >= rows for t in (inp, in32, z, gate, out)), "delta: inputs")
    kc, vc = s.kv_heads * s.dim, s.heads * s.vdim
    _req(inp.shape[1] >= max(cols[0] + kc, cols[1] + kc, cols[2] + vc) and in32.shape[1] >= ob + s.heads
         and z.shape[1] >= s.heads * s.dim and min(gate.shape[1], out.shape[1]) >= vc, "delta: columns")
    _req((runs is None) != (slot is None), "delta: runs or rows")
    _req(table.dtype == torch.int32 and table.shape[0] <= S.shape[0], "delta: page table")
    for t in (runs, slot, pos):
        _req(t is None or (t.dtype == torch.int32 and t.is_contiguous()), "delta: int32 rows")
    q = {n: _p(t) for n, t in (("runs", runs), ("slot", slot), ("pos", pos))}
    dk, dv = s.state_dims
    return DeltaArgs(_p(inp), _p(in32), _p(z), _p(gate), _p(w["conv"]), _p(w["decay"]), _p(w["dt_bias"]), _p(w["norm"]),
                     _p(S), _p(ring), q["runs"], q["slot"], q["pos"], _p(table), _p(out), inp.stride(0), in32.stride(0),
                     z.stride(0), gate.stride(0), out.stride(0), *cols, ob, s.heads, s.kv_heads, s.dim, s.vdim, s.taps,
                     dk, dv, table.shape[1], n_pages, float(s.q_scale), float(s.unit_eps), float(eps))


def check_runs(runs_host, rows: int, slots: int) -> None:
    """Runs inside the batch, one per slot (a state has one writer)."""
    r0, n, sl, p0 = (runs_host[:, i] for i in range(4))
    _req(bool((n >= 1).all() and (r0 >= 0).all() and (p0 >= 0).all() and (sl >= 0).all()) and int((r0 + n).max()) <= rows
         and int(sl.max()) < slots, "delta runs: rows")
    _req(len(set(sl.tolist())) == sl.numel(), "delta runs: one run per slot and step")


def steps(a: DeltaArgs, dtype, n: int, keep: bool) -> None:
    """n runs step by step. ``keep``: all of one row, their inputs join the ring here (else :func:`ring` follows)."""
    _check(lib().lsa_delta_steps(is_f32(dtype), ctypes.byref(a), n, int(keep), _stream()), "lsa_delta_steps")


def ring(a: DeltaArgs, dtype, n: int) -> None:
    _check(lib().lsa_delta_ring(is_f32(dtype), ctypes.byref(a), n, _stream()), "lsa_delta_ring")


CHUNK = 32  # rows per chunk (C in csrc/kernels/delta_chunk.hip)


def chunk_bytes(s) -> int:
    """Workspace bytes of one (chunk, head); 0: the chunked kernels do not take this size."""
    return int(lib().lsa_delta_chunk_bytes(*s.state_dims))


def chunk_groups(runs: list, most: int) -> list:
    """Long runs (row0, rows, slot, pos0) cut into groups of at most ``most`` chunks, each run going on in the next
    group where it stopped: [(chunks int32 [n, 8], spans int32 [m, 8])], host."""
    at, groups = [0] * len(runs), []
    while True:
        live = [i for i, r in enumerate(runs) if at[i] < r[1]][:most]
        if not live:
            return groups
        share, chunks, spans = max(1, most // len(live)), [], []
        for i in live:
            row0, n, slot, pos0 = runs[i]
            take = min(n - at[i], share * CHUNK)
            spans.append([len(chunks), -(-take // CHUNK), slot, pos0 + at[i], row0 + at[i], take, 0, 0])
            for c in range(0, take, CHUNK):
                b = at[i] + c
                chunks.append([row0 + b, min(CHUNK, take - c), slot, pos0 + b, b, 0, 0, 0])
            at[i] += take
        groups.append((torch.tensor(chunks, dtype=torch.int32), torch.tensor(spans, dtype=torch.int32)))


def chunked(a: DeltaArgs, chunks, spans, ws, nbytes: int, o32) -> None:
    """One group of :func:`chunk_groups` of checked runs (tables on the device), bf16. ``ws``: bytes; ``o32`` fp32
    [rows, heads vdim]."""
    _req(o32.dtype == torch.float32 and o32.is_contiguous() and o32.dim() == 2 and o32.shape[1] == a.heads * a.vdim,
         "delta: read-outs")
    _req(all(t.dtype == torch.int32 and t.is_contiguous() and t.shape[1] == 8 for t in (chunks, spans)), "delta: tables")
    _req(ws.dtype == torch.uint8 and ws.numel() >= chunks.shape[0] * a.heads * nbytes and nbytes > 0, "delta: workspace")
    _check(lib().lsa_delta_chunked(ctypes.byref(a), _p(chunks), chunks.shape[0], _p(spans), spans.shape[0], _p(ws),
                                   _p(o32), _stream()), "lsa_delta_chunked")


def declare(L: ctypes.CDLL) -> None:
    """Signatures of these entry points (called by hip.load_library)."""
    vp, i = ctypes.c_void_p, ctypes.c_int
    da = ctypes.POINTER(DeltaArgs)
    hip.set_signatures(L, {
        "lsa_delta_steps": [i, da, i, i, vp],
        "lsa_delta_ring": [i, da, i, vp],
        "lsa_delta_chunk_bytes": [i, i],
        "lsa_delta_chunked": [da, vp, i, vp, i, vp, vp, vp],
    })
