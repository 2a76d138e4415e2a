"""Bindings and weights of the latent-attention kernels (csrc/kernels/latent*.hip).

The conventions of :mod:`.hip` hold: shapes are checked on the host, launches go to torch's current
stream, nothing falls back to another implementation."""
from __future__ import annotations

import ctypes
from typing import Optional

import torch

from . import hip
from .hip import _check, _p, _req, _stream, lib
from .packing import pack_b
from .stream import (Linear, cast_rows, is_f32, logits_argmax, pad2, stream_add_norm, stream_embed,  # noqa: F401
                     stream_norm)

PAGE = 64  # tokens per cache page (LAT_PAGE in csrc/kernels/latent.h)


class LatentArgs(ctypes.Structure):
    _fields_ = ([(n, ctypes.c_void_p) for n in ("cache", "table", "slot", "pos", "index", "cos_t", "sin_t", "sink")]
                + [(n, ctypes.c_int) for n in ("max_pages", "n_pages", "window", "heads", "dim", "rot_dim", "rot_dims", "vdim",
                                               "kv_rank", "q_rank", "dkp", "rp", "dvp", "krp")]
                + [("scale", ctypes.c_float), ("eps", ctypes.c_float)])


# ------------------------------------------------------------------------------ latent attention
def tuned_size(s) -> bool:
    """The MFMA kernels of the absorbed form take this size (others run the plain kernels)."""
    return s.krp in (64, 128, 256, 512) and s.rp == 64


def expand_size(s) -> bool:
    """The MFMA kernel of the expanded form takes this size."""
    return s.rp == 64 and s.dkp in (64, 128) and s.dvp in (64, 128)


def head_groups(s) -> int:
    """Workgroups per (row, split) of attend_mfma: head tiles of 16, 1 / 2 / 4 to a workgroup (at
    most 2 with 512-wide latents)."""
    tiles = -(-s.heads // 16)
    per = tiles if tiles < 3 else (2 if s.krp == 512 else 4)
    return -(-tiles // per)


def pack_heads(w: torch.Tensor) -> torch.Tensor:
    """Per-head matrices [H, N, K] (N % 16, K % 32) in MFMA fragment order, head after head."""
    return pack_b(w.reshape(-1, w.shape[2])).contiguous()


def prefill_tile_rows(rows: int, heads: int) -> int:
    """Query rows per tile of the expanded form: 128, halved while the chip would idle."""
    t = 128
    while t > 16 and -(-rows // t) * heads < hip.N_CU:
        t //= 2
    return t


def make_args(spec, cache, table, slot, pos, cos, sin, eps: float, index=None, sink=None) -> LatentArgs:
    """``cache`` [pages, PAGE, krp + rp], ``table`` int32 [slots, max_pages], ``slot`` / ``pos`` int32
    [rows], ``cos`` / ``sin`` fp32 [>= max_pages * PAGE, rot_dims / 2], ``index`` int32 [entries], ``sink`` fp32 [heads] in log2 units."""
    _req(cache.dim() == 3 and cache.shape[1] == PAGE and cache.shape[2] == spec.cache_width and cache.is_contiguous()
         and cache.is_cuda, "latent: cache [pages, 64, width]")
    _req(table.dtype == torch.int32 and table.dim() == 2 and table.is_contiguous(), "latent: int32 page table")
    _req(slot.dtype == torch.int32 and pos.dtype == torch.int32, "latent: int32 slot / pos")
    _req(index is None or index.dtype == torch.int32, "latent: int32 index")
    _req(cos.dtype == torch.float32 and cos.shape == sin.shape and cos.shape[0] >= table.shape[1] * PAGE
         and cos.shape[1] == spec.rot_dims // 2, "latent: rotation tables")
    _req((sink is not None) == spec.sink and (sink is None or (sink.dtype == torch.float32 and sink.numel() == spec.heads
                                                               and sink.is_contiguous())), "latent: sink")
    return LatentArgs(cache.data_ptr(), table.data_ptr(), slot.data_ptr(), pos.data_ptr(),
                      None if index is None else index.data_ptr(), cos.data_ptr(), sin.data_ptr(), _p(sink),
                      table.shape[1], cache.shape[0], spec.window, spec.heads, spec.dim, spec.rot_dim, spec.rot_dims, spec.vdim, spec.kv_rank,
                      spec.q_rank, spec.dkp, spec.rp, spec.dvp, spec.krp, float(spec.scale), float(eps))


def append(a: LatentArgs, rows: int, inp, oq: int, ok: int, gq, gk, cq) -> None:
    _req(inp.dtype == cq.dtype and min(inp.shape[0], cq.shape[0]) >= rows and cq.shape[1] >= a.q_rank, "append: shapes")
    _req(gq.dtype == torch.float32 and gq.numel() >= a.q_rank and gk.numel() >= a.kv_rank, "append: norm weights")
    _check(lib().lsa_latent_append(is_f32(inp.dtype), ctypes.byref(a), rows, _p(inp), inp.stride(0), oq, ok, _p(gq),
                                   _p(gk), _p(cq), cq.stride(0), _stream()), "lsa_latent_append")


def absorb(a: LatentArgs, n: int, q, wk, qt) -> None:
    cw = a.krp + a.rp
    _req(q.dtype == wk.dtype == qt.dtype and wk.numel() == a.heads * a.dkp * a.krp and qt.numel() >= n * a.heads * cw
         and qt.is_contiguous(), "absorb: shapes")
    _check(lib().lsa_latent_absorb(is_f32(q.dtype), ctypes.byref(a), n, _p(q), q.stride(0), _p(wk), _p(qt), _stream()),
           "lsa_latent_absorb")


def attend(a: LatentArgs, n: int, qt, ns: int, po, pm) -> None:
    e = n * a.heads * ns
    _req(po.dtype == pm.dtype == torch.float32 and po.numel() >= e * a.krp and pm.numel() >= 2 * e, "attend: workspace")
    _req(qt.numel() >= n * a.heads * (a.krp + a.rp), "attend: query shape")
    _check(lib().lsa_latent_attend(is_f32(qt.dtype), ctypes.byref(a), n, _p(qt), ns, _p(po), _p(pm), _stream()),
           "lsa_latent_attend")


def value(a: LatentArgs, n: int, po, pm, ns: int, wv, gate, out) -> None:
    """``gate``: a column view of the input projection whose first column is the gate's, or None."""
    e = n * a.heads * ns
    _req(po.numel() >= e * a.krp and pm.numel() >= 2 * e and wv.numel() == a.heads * a.krp * a.dvp
         and out.shape[1] >= a.heads * a.dvp and wv.dtype == out.dtype, "value: shapes")
    _req(gate is None or (gate.dtype == out.dtype and gate.shape[1] >= a.heads * a.dvp), "value: gate")
    _check(lib().lsa_latent_value(is_f32(out.dtype), ctypes.byref(a), n, _p(po), _p(pm), ns, _p(wv), _p(gate),
                                  0 if gate is None else gate.stride(0), _p(out), out.stride(0), _stream()),
           "lsa_latent_value")


def absorb_mfma(a: LatentArgs, n: int, q, wk, qt) -> None:
    """As :func:`absorb` in bf16; ``wk``: pack_heads of [heads, krp, dkp]."""
    _req(q.dtype == wk.dtype == qt.dtype == torch.bfloat16 and wk.numel() == a.heads * a.dkp * a.krp
         and qt.numel() >= n * a.heads * (a.krp + a.rp) and qt.is_contiguous(), "absorb_mfma: shapes")
    _check(lib().lsa_latent_absorb_mfma(ctypes.byref(a), n, _p(q), q.stride(0), _p(wk), _p(qt), _stream()),
           "lsa_latent_absorb_mfma")


def attend_mfma(a: LatentArgs, n: int, qt, ns: int, po, pm) -> None:
    e = n * a.heads * ns
    _req(qt.dtype == torch.bfloat16 and qt.numel() >= n * a.heads * (a.krp + a.rp), "attend_mfma: query shape")
    _req(po.dtype == pm.dtype == torch.float32 and po.numel() >= e * a.krp and pm.numel() >= 2 * e,
         "attend_mfma: workspace")
    _check(lib().lsa_latent_attend_mfma(ctypes.byref(a), n, _p(qt), ns, _p(po), _p(pm), _stream()),
           "lsa_latent_attend_mfma")


def value_mfma(a: LatentArgs, n: int, po, pm, ns: int, wv, gate, out) -> None:
    """As :func:`value` in bf16; ``wv``: pack_heads of [heads, dvp, krp]."""
    e = n * a.heads * ns
    _req(po.numel() >= e * a.krp and pm.numel() >= 2 * e and wv.numel() == a.heads * a.krp * a.dvp
         and out.shape[1] >= a.heads * a.dvp and wv.dtype == out.dtype == torch.bfloat16, "value_mfma: shapes")
    _req(gate is None or (gate.dtype == out.dtype and gate.shape[1] >= a.heads * a.dvp), "value_mfma: gate")
    _check(lib().lsa_latent_value_mfma(ctypes.byref(a), n, _p(po), _p(pm), ns, _p(wv), _p(gate),
                                       0 if gate is None else gate.stride(0), _p(out), out.stride(0), _stream()),
           "lsa_latent_value_mfma")


def gather(a: LatentArgs, src, n: int, out) -> None:
    """Cached entries of the (slot, position) pairs ``src`` int32 [n, 2] -> rows of ``out`` (bf16)."""
    _req(src.dtype == torch.int32 and src.is_contiguous() and src.numel() >= 2 * n and out.dtype == torch.bfloat16
         and out.shape[0] >= n and out.shape[1] == a.krp + a.rp and out.is_contiguous(), "gather: shapes")
    _check(lib().lsa_latent_gather(ctypes.byref(a), _p(src), n, _p(out), _stream()), "lsa_latent_gather")


_TILES_OK = None  # the last tile table prefill() validated: a forward checks its table once, not per layer


def prefill(a: LatentArgs, tiles, tiles_host, q, kv, lat, gate, out, rows: int, tokens: int) -> None:
    """Attention of the query tiles [row0, nrows, kv0, pos0, kvlen, base, 0, 0] over expanded keys and
    values ``kv`` [tokens, heads (dkp + dvp)] and the gathered entries ``lat`` [tokens, krp + rp], the
    sequence's from row kv0 (position ``base``) on."""
    _req(all(t.dtype == torch.bfloat16 for t in (q, kv, lat, out)) and tiles.dtype == torch.int32
         and tiles.shape == tiles_host.shape and tiles.shape[1] == 8 and tiles.is_contiguous(), "prefill: types")
    _req(min(q.shape[0], out.shape[0]) >= rows and out.shape[1] >= a.heads * a.dvp
         and min(kv.shape[0], lat.shape[0]) >= tokens and kv.shape[1] >= a.heads * (a.dkp + a.dvp)
         and lat.shape[1] == a.krp + a.rp and lat.is_contiguous(), "prefill: shapes")
    _req(gate is None or (gate.dtype == torch.bfloat16 and gate.shape[0] >= rows
                          and gate.shape[1] >= a.heads * a.dvp), "prefill: gate")
    global _TILES_OK
    key = (tiles.data_ptr(), rows, tokens, a.max_pages)
    if not (_TILES_OK is not None and _TILES_OK[0] is tiles_host and _TILES_OK[1] == key):
        r0, nr, k0, p0, kl, base = (tiles_host[:, i] for i in range(6))
        _req(bool((nr >= 1).all() and (nr <= 128).all() and (r0 >= 0).all()) and int((r0 + nr).max()) <= rows,
             "prefill: tile rows")
        _req(bool((k0 >= 0).all() and (kl >= 1).all() and (p0 >= 0).all()) and int((k0 + kl).max()) <= tokens
             and bool((base >= 0).all() and (p0 >= base).all() and (p0 + nr <= base + kl).all())
             and int((base + kl).max()) <= a.max_pages * PAGE, "prefill: tile keys")
        _TILES_OK = (tiles_host, key)
    _check(lib().lsa_latent_prefill(ctypes.byref(a), _p(tiles), tiles.shape[0], _p(q), q.stride(0), _p(kv), kv.stride(0),
                                    _p(lat), _p(gate), 0 if gate is None else gate.stride(0), _p(out), out.stride(0),
                                    _stream()), "lsa_latent_prefill")


def declare(L: ctypes.CDLL) -> None:
    """Signatures of these entry points (called by hip.load_library)."""
    vp, i, f = ctypes.c_void_p, ctypes.c_int, ctypes.c_float
    la = ctypes.POINTER(LatentArgs)
    hip.set_signatures(L, {
        "lsa_latent_append": [i, la, i, vp, i, i, i, vp, vp, vp, i, vp],
        "lsa_latent_absorb": [i, la, i, vp, i, vp, vp, vp],
        "lsa_latent_attend": [i, la, i, vp, i, vp, vp, vp],
        "lsa_latent_value": [i, la, i, vp, vp, i, vp, vp, i, vp, i, vp],
        "lsa_latent_absorb_mfma": [la, i, vp, i, vp, vp, vp],
        "lsa_latent_attend_mfma": [la, i, vp, i, vp, vp, vp],
        "lsa_latent_value_mfma": [la, i, vp, vp, i, vp, vp, i, vp, i, vp],
        "lsa_latent_prefill": [la, vp, i, vp, i, vp, i, vp, vp, i, vp, i, vp],
        "lsa_latent_gather": [la, vp, i, vp, vp],
    })
