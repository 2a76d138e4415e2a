"""Bindings and weights of the mixture-of-experts kernels (csrc/kernels/moe.hip).

The conventions of :mod:`.hip` hold: shapes are checked on the host, launches go to torch's current
stream, nothing falls back to another implementation."""
from __future__ import annotations

import ctypes

import torch

from . import hip
from .hip import _check, _p, _req, _stream, lib
from .packing import fuse_gate_up, pack_b
from .stream import is_f32, pad2


def pad128(n: int) -> int:
    return -(-n // 128) * 128


class Experts:
    """The experts' products, one after another: gate and up interleaved by 16 rows [E][2 ff][width] and down
    [E][width][ff], sizes padded to 128; bf16 weights packed for the MFMA kernels."""

    def __init__(self, gate: list, up: list, down: list):
        self.ff, self.width = pad128(gate[0].shape[0]), pad128(gate[0].shape[1])
        self.f32 = is_f32(gate[0].dtype)
        lay = (lambda w: w.contiguous()) if self.f32 else (lambda w: pack_b(w).contiguous())
        self.up = torch.stack([lay(fuse_gate_up(pad2(g, self.ff, self.width), pad2(u, self.ff, self.width)))
                               for g, u in zip(gate, up)])
        self.down = torch.stack([lay(pad2(d, self.width, self.ff)) for d in down])
        self.experts = len(gate)

    def tensors(self) -> list:
        return [self.up, self.down]


def tile_rows(pairs: int, experts: int, f32: bool) -> int:
    """Pairs per tile: what an expert gets on average, rounded to a kernel's size."""
    if f32:
        return 64
    mean = pairs / experts  # (a second tile of an expert reads its weights again)
    return next((n for n in (16, 32, 64) if mean <= 0.75 * n), 128 if mean <= 320 else 256)


def max_tiles(pairs: int, experts: int, rows: int) -> int:
    return min(experts, pairs) + pairs // rows


def route(logits, rows: int, experts: int, top: int, expert, weight) -> None:
    """fp32 router logits -> chosen experts and their softmax weights [rows * top]."""
    _req(logits.dtype == torch.float32 and logits.stride(1) == 1 and logits.shape[0] >= rows
         and logits.shape[1] >= experts, "route: logits")
    _req(expert.dtype == torch.int32 and weight.dtype == torch.float32 and min(expert.numel(), weight.numel()) >= rows * top,
         "route: outputs")
    _check(lib().lsa_moe_route(_p(logits), logits.stride(0), rows, experts, top, _p(expert), _p(weight), _stream()),
           "lsa_moe_route")


def group(expert, pairs: int, experts: int, rows: int, order, place, tiles) -> int:
    """Pairs sorted by expert (``order``; ``place`` is its inverse) and their tiles; returns the table's length."""
    n = max_tiles(pairs, experts, rows)
    _req(all(t.dtype == torch.int32 for t in (expert, order, place, tiles)) and tiles.numel() >= 4 * n
         and min(expert.numel(), order.numel(), place.numel()) >= pairs, "group: shapes")
    _check(lib().lsa_moe_group(_p(expert), pairs, experts, rows, n, _p(order), _p(place), _p(tiles), _stream()),
           "lsa_moe_group")
    return n


def route_group(logits, rows: int, experts: int, top: int, tile: int, expert, weight, order, place, tiles) -> int:
    """:func:`route` and :func:`group`, in one launch where there are few rows."""
    pairs = rows * top
    if rows > 16 or experts > 256:
        route(logits, rows, experts, top, expert, weight)
        return group(expert, pairs, experts, tile, order, place, tiles)
    n = max_tiles(pairs, experts, tile)
    _req(logits.dtype == torch.float32 and logits.stride(1) == 1 and logits.shape[0] >= rows
         and logits.shape[1] >= experts and weight.dtype == torch.float32 and weight.numel() >= pairs, "route: shapes")
    _req(all(t.dtype == torch.int32 for t in (expert, order, place, tiles)) and tiles.numel() >= 4 * n
         and min(expert.numel(), order.numel(), place.numel()) >= pairs, "group: shapes")
    _check(lib().lsa_moe_route_group(_p(logits), logits.stride(0), rows, experts, top, _p(expert), _p(weight), tile, n,
                                     _p(order), _p(place), _p(tiles), _stream()), "lsa_moe_route_group")
    return n


def gemm(tiles, n_tiles: int, rows: int, order, top: int, a, w, n: int, k: int, out, pairs: int, glu: bool) -> None:
    """One product of every tile's expert: ``glu`` up from rows of h (``a``) to out [pairs, n / 2], else down from
    out rows of the sorted pairs (``a`` [pairs, k]) to out [pairs, n]."""
    _req(a.dtype == w.dtype == out.dtype and a.stride(1) == 1 and a.shape[1] >= k and out.stride(1) == 1
         and out.shape[0] >= pairs and out.shape[1] >= (n // 2 if glu else n) and order.numel() >= pairs
         and (a.shape[0] * top >= pairs if glu else a.shape[0] >= pairs), "moe: shapes")
    _req(w[0].numel() == n * k and w.is_contiguous(), "moe: weights")
    if rows > 64:
        _check(lib().lsa_moe_gemm_big(int(glu), _p(tiles), n_tiles, rows, _p(order), top, _p(a), a.shape[0] if glu else 0,
                                      a.stride(0), _p(w), n, k, _p(out), out.stride(0), _stream()), "lsa_moe_gemm_big")
        return
    _check(lib().lsa_moe_gemm(is_f32(a.dtype), int(glu), _p(tiles), n_tiles, rows, _p(order), top, _p(a), a.stride(0), _p(w),
                              n, k, _p(out), out.stride(0), _stream()), "lsa_moe_gemm")


def declare(L: ctypes.CDLL) -> None:
    """Signatures of these entry points (called by hip.load_library)."""
    vp, i = ctypes.c_void_p, ctypes.c_int
    hip.set_signatures(L, {
        "lsa_moe_route": [vp, i, i, i, i, vp, vp, vp],
        "lsa_moe_group": [vp, i, i, i, i, vp, vp, vp, vp],
        "lsa_moe_route_group": [vp, i, i, i, i, vp, vp, i, i, vp, vp, vp, vp],
        "lsa_moe_gemm_big": [i, vp, i, i, vp, i, vp, i, i, vp, i, i, vp, i, vp],
        "lsa_moe_gemm": [i, i, vp, i, i, vp, i, vp, i, vp, i, i, vp, i, vp],
    })
