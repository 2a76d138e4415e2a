"""StackEngine: a pipeline stage of a config-driven layer stack (:class:`..models.stack.StackConfig`).

The same step function, sequence API, decode graphs and serving as :class:`.engine.StageEngine`, for
decoders that differ from Llama / GPT-2 in what a layer is made of:

* the residual stream is fp32 (rows of ``hidden_dtype``), or several streams side by side; how the sublayers read
  and join it is the layer's block (:mod:`.blocks`);
* mixers and feed-forwards come from the layer's spec; layers may share tensors, or read another
  layer's keys and values;
* the cache is paged (:mod:`.paging`): one pool for all slots, one page table for all layers;
* recurrent layers keep a state per slot, which starts from zero at position 0;
* layers that run several times in a row are as many entries of the stack, with one layer's weights and caches
  of their own; what a pass starts from reads the embedding output, so they begin on the first stage;
* projections run the framework's GEMV / GEMM kernels on padded weights (ops/stream.Linear); fp32
  engines run every product in true fp32.
"""
from __future__ import annotations

from typing import Optional

import torch
import torch.nn.functional as F

from ..config import ceil_div
from ..models.stack import (AttentionSpec, DeltaSpec, LatentSpec, MlstmSpec, PairSpec, RetentionSpec, StackConfig, leaves,
                            pad_to)
from .attn_mixer import rotary_tables
from .blocks import COPY, Entry, Layer, Sum, block
from .engine import StageEngine, WeightSource
from .latent_mixer import rotation_tables
from .paging import PagePool
from .plan import Plan

PAGE = 64


def embed_rows(cfg: StackConfig, table: torch.Tensor, ids: torch.Tensor) -> torch.Tensor:
    """Rows of the stream for ``ids`` [n], without an engine (an ingress that holds the table only)."""
    h = torch.empty((ids.numel(), cfg.stream_width), dtype=torch.float32, device=table.device)
    if table.device.type != "cuda":
        return h.copy_((F.embedding(ids.long(), table).float() * cfg.embed_scale).repeat(1, cfg.streams))
    from ..ops import stream as L
    L.stream_embed(ids.to(torch.int32), table, cfg.embed_scale, h, None, ids.numel(), cfg.streams)
    return h


class StackEngine(StageEngine):
    GPU_DTYPES = (torch.bfloat16, torch.float32)
    SCRATCH_ATTRS = ("buf_h", "buf_x", "buf_y", "flat", "qt", "part_o", "part_ml", "coop_ws", "sk_ws", "keys", "tokens",
                     "_x_ready")
    # rows from which a run of one sequence's consecutive positions attends in the expanded form: below,
    # multiplying keys and values out costs more than the wider products of the absorbed form
    expand_min = 64

    def __init__(self, cfg: StackConfig, start: int, end: int, device="cpu", dtype=torch.bfloat16, *,
                 has_embed: bool = False, has_head: bool = False, source: Optional[WeightSource] = None,
                 max_slots: int = 1, max_seq: int = 2048, max_prefill_rows: int = 2048, causal: bool = True,
                 load: bool = True, verbose: bool = False, head_cols: Optional[tuple] = None,
                 weight_dtype: str = "bf16", cache_tokens: Optional[int] = None):
        """``cache_tokens``: tokens the page pool holds (default: every slot's longest sequence)."""
        if not causal:
            raise ValueError("stack engines attend causally")
        if weight_dtype != "bf16":
            raise ValueError("stack engines keep their weights in the compute type (weight_dtype='bf16')")
        pages = ceil_div(min(max_seq, cfg.max_position_embeddings), PAGE) * max_slots
        self.cache_pages = pages if cache_tokens is None else ceil_div(cache_tokens, PAGE)
        self._rot: dict = {}
        self._expand_bufs: dict = {}
        self._workspaces: dict = {}
        super().__init__(cfg, start, end, device, dtype, has_embed=has_embed, has_head=has_head, source=source,
                         max_slots=max_slots, max_seq=max_seq, max_prefill_rows=max_prefill_rows, causal=causal,
                         load=load, verbose=verbose, head_cols=head_cols, weight_dtype=weight_dtype)

    # ------------------------------------------------------------------------- loading
    def _init_routes(self) -> None:
        pass

    @property
    def hidden_dtype(self) -> torch.dtype:
        return torch.float32

    @property
    def head_vocab(self) -> int:
        """Vocabulary entries this stage's part of the head covers."""
        return min(self.head_v1, self.cfg.vocab_size) - self.head_v0

    @property
    def width_p(self) -> int:
        return pad_to(self.cfg.hidden_size, 128)

    def load(self) -> None:
        cfg, dev, dt = self.cfg, self.device, self.dtype
        if self.source is None:
            raise ValueError("StackEngine needs a WeightSource")
        self.layers, shared = [], {}
        for i in range(self.start, self.end):
            spec = cfg.layers[i]
            if spec.owner not in shared:
                self._log(f"[INFO] loading layer {i}")
                shared[spec.owner] = block(cfg, spec, self.source.layer(i, dev, dt), self.gpu)
            self.layers.append(Layer(spec, shared[spec.owner]))
        self.loop = None
        if any(l.spec.enters is not None for l in self.layers):
            if self.start:
                raise ValueError("layers that read the embedding output belong on the first stage")
            self.loop = Entry(cfg, self.source.extra(dev, dt), self.gpu)
        if self.has_embed:
            self.embed_w = self.source.embedding(dev, dt).contiguous()
        if self.has_head:
            self.final_norm = (self.source.final_norm(dev, dt).float().reshape(-1)
                               + cfg.norm_offset).expand(cfg.hidden_size).contiguous()
            if cfg.logit_scale != 1.0:  # the head is linear: its input is scaled
                self.final_norm = self.final_norm * cfg.logit_scale
            self.head_read = Sum(torch.ones(cfg.streams, device=dev), self.final_norm)
            head = self.embed_w if cfg.tie_word_embeddings and self.has_embed else self.source.lm_head(dev, dt)
            head = F.pad(head, (0, 0, 0, cfg.head_rows - cfg.vocab_size))[self.head_v0:self.head_v1]
            if self.gpu:
                from ..ops import stream as L
                self.lm_head = L.Linear(head)
            else:
                self.lm_head = head.contiguous()
            n = self.lm_head.n if self.gpu else head.shape[0]
            if n > self.head_vocab:  # padding rows must not win the argmax
                self.head_bias = torch.zeros(n, dtype=torch.float32, device=dev)
                self.head_bias[self.head_vocab:] = -3.0e38
        self._alloc_runtime()

    # ------------------------------------------------------------------------- memory
    def _alloc_runtime(self) -> None:
        cfg, dev, dt = self.cfg, self.device, self.dtype
        self.pool = PagePool(self.cache_pages, self.max_slots, self.max_seq, PAGE, dev)
        mixers = [m for l in self.layers for m in leaves(l.spec.mixer)]
        # tables of pooled blocks, by tokens per block: their pages follow those of the tokens
        self.pools = {p: PagePool(self._pooled_pages(p), self.max_slots, self.max_seq, PAGE * p, dev)
                      for p in sorted({getattr(m, "pool", 0) for m in mixers} - {0})}

        self.k_cache, self.v_cache, self.states, self.pooled = [], [], [], []
        for i, l in enumerate(self.layers):
            k, v, state, pooled = self._layer_memory(l.spec.mixer)
            self.pooled.append(pooled)
            j = getattr(l.spec.mixer, "kv_from", None)
            if j is not None:
                if j < self.start:
                    raise ValueError(f"layer {self.start + i} reads layer {j}'s keys and values: both belong on one stage")
                k, v = self.k_cache[j - self.start], self.v_cache[j - self.start]
            self.k_cache.append(k)
            self.v_cache.append(v)
            self.states.append(state)
        for m in mixers:
            if isinstance(m, LatentSpec) and (m.rot_base, m.rot_dims) not in self._rot:
                self._rot[(m.rot_base, m.rot_dims)] = rotation_tables(m, self.pool.max_pages * PAGE, dev)
            elif getattr(m, "rot", None) is not None and m.rot not in self._rot:
                self._rot[m.rot] = rotary_tables(m.rot, self.pool.max_pages * PAGE, dev)
        self.cos = self.sin = None
        if self.gpu:
            # widest row of every intermediate over the layers, and its type
            self._widths = {"y2": (self.width_p if cfg.hidden_size % 16 else 0, torch.float32)}
            for l in [x.w for x in self.layers] + ([self.loop] if self.loop is not None else []):
                for part in l.scratch():
                    for k, n in part.items():
                        n, t = n if isinstance(n, tuple) else (n, dt)
                        self._widths[k] = (max(self._widths.get(k, (0,))[0], n), t)
            for k, v in self._scratch_set(max(self.max_prefill_rows, self.DECODE_MAX_ROWS)).items():
                setattr(self, k, v)

    def _layer_memory(self, m) -> tuple:
        """(key cache, value cache, state, pooled keys and values) of one layer's mixer; latent attention has one
        cache."""
        dev, dt, pages = self.device, self.dtype, self.cache_pages
        if isinstance(m, PairSpec):
            (k, v, _, pooled), (_, _, state, _) = (self._layer_memory(x) for x in (m.left, m.right))
            return k, v, state, pooled
        if isinstance(m, LatentSpec):
            width = m.cache_width if self.gpu else m.kv_rank + m.rot_dim
            return torch.zeros((pages, PAGE, width), dtype=dt, device=dev), None, None, ()
        if isinstance(m, RetentionSpec):
            dims = m.state_dims if self.gpu else (m.dim, m.vdim)
            return None, None, (torch.zeros((self.max_slots, m.heads) + dims, dtype=torch.float32, device=dev),), ()
        if isinstance(m, MlstmSpec):
            dims, n = (m.state_dims, m.copies) if self.gpu else ((m.dim, m.vdim), 1)
            shapes = (dims, (n, dims[0]), (n,))
            return None, None, tuple(torch.zeros((self.max_slots, m.heads) + s, dtype=torch.float32, device=dev) for s in shapes), ()
        if isinstance(m, DeltaSpec):
            from ..ops.delta import state_shapes
            S, ring = state_shapes(m, self.max_slots)
            if not self.gpu:
                S = S[:2] + (m.dim, m.vdim)
            return None, None, tuple(torch.zeros(n, dtype=torch.float32, device=dev) for n in (S, ring)), ()
        if m.kv_from is not None:
            return None, None, None, ()
        from ..ops.paged_attn import cache_shapes

        def cache(n):
            shapes = cache_shapes(m, n) if self.gpu else ((n, PAGE, m.kv_heads, m.dim), (n, PAGE, m.kv_heads, m.vdim))
            return tuple(torch.zeros(x, dtype=dt, device=dev) for x in shapes)
        return cache(pages) + (None, cache(self._pooled_pages(m.pool)) if m.pool else ())

    def _pooled_pages(self, pool: int) -> int:
        """Pages of pooled blocks: never short while there are pages of tokens."""
        from ..ops.paged_attn import pooled_pages
        return pooled_pages(self.cache_pages, self.max_slots, pool)

    def cache(self, i: int) -> tuple:
        """Caches of layer i of this stage: keys, values, and those of its pooled blocks."""
        return (self.k_cache[i], self.v_cache[i]) + self.pooled[i]

    @property
    def carries_state(self) -> bool:
        """Running a token twice is not the same as once (a recurrent layer's state moves on)."""
        return any(s is not None for s in self.states)

    def _projections(self) -> list:
        out = []
        for l in self.layers:
            gated = [p for p in (getattr(l.mlp, k, None) for k in ("gate_up", "shared_glu")) if p is not None]
            out += [(p.n, p.k, any(p is g for g in gated)) for p in l.w.projections()]
        if self.loop is not None:
            out.append((self.loop.lin.n, self.loop.lin.k, False))
        if self.has_head:
            out.append((self.lm_head.n, self.lm_head.k, False))
        return sorted(set(out))

    def _scratch_set(self, R: int) -> dict:
        """Everything a forward of up to R rows writes besides the cache."""
        from ..ops import hip, packing
        dev, dt, W = self.device, self.dtype, self.width_p
        out = {"buf_h": torch.zeros((R, self.cfg.stream_width), dtype=torch.float32, device=dev),
               "buf_x": torch.zeros((R, W), dtype=dt, device=dev),
               "buf_y": torch.zeros((R, W), dtype=torch.float32, device=dev),
               "flat": {k: torch.zeros(R * n, dtype=t, device=dev) for k, (n, t) in self._widths.items() if n},
               "keys": torch.zeros(R, dtype=torch.int64, device=dev),
               "tokens": torch.zeros(R, dtype=torch.int32, device=dev), "_x_ready": False, "coop_ws": None, "sk_ws": None}
        # attention split over keys: absorbed queries and split partials of up to ATTEND_ITEMS (row, split)
        # pairs at a time
        items = self.ATTEND_ITEMS
        ms = [m for l in self.layers for m in leaves(l.spec.mixer)]
        latent, paged = ([m for m in ms if isinstance(m, t)] for t in (LatentSpec, AttentionSpec))
        qn = max((m.heads * m.cache_width for m in latent), default=0)
        on = max([m.heads * m.krp for m in latent] + [m.heads * m.dvp for m in paged], default=0)
        hn = max((m.heads for m in latent + paged), default=0)
        out["qt"] = torch.zeros(items * qn, dtype=dt, device=dev)
        out["part_o"] = torch.zeros(items * on, dtype=torch.float32, device=dev)
        out["part_ml"] = torch.zeros(items * hn * 2, dtype=torch.float32, device=dev)
        if dt == torch.bfloat16:
            shapes = self._projections()
            floats, groups = packing.coop_workspace_need([(n, k) for n, k, _ in shapes], self.DECODE_MAX_ROWS,
                                                         even_n=[(n, k) for n, k, even in shapes if even])
            out["coop_ws"] = hip.CoopWorkspace(dev, slab_floats=max(floats, 1 << 20), groups=max(groups, 4096))
            out["sk_ws"] = hip.SkWorkspace(dev)
        return out

    ATTEND_ITEMS = 1024  # (row, key split) pairs of one absorbed-attention launch

    def decode_scratch(self, k: int, rows: Optional[int] = None) -> dict:
        if k == 0:
            return {a: getattr(self, a) for a in self.SCRATCH_ATTRS}
        R = max(self.DECODE_MAX_ROWS, rows or 0)
        if k in self._scratch and self._scratch[k]["buf_h"].shape[0] < R:
            raise ValueError(f"scratch set {k} was allocated for fewer than {R} rows")
        if k not in self._scratch:
            self._scratch[k] = self._scratch_set(R)
        return self._scratch[k]

    def scratch_view(self, name: str, rows: int, n: int) -> torch.Tensor:
        return self.flat[name][:rows * n].view(rows, n)

    def attend_scratch(self) -> tuple:
        """(absorbed queries, partial sums, partial max / sum)."""
        return self.qt, self.part_o, self.part_ml

    def expand_scratch(self, s, tokens: int, n: int) -> tuple:
        """Gathered latents and expanded keys / values (grown on demand: long portions run eagerly;
        one set per stream of concurrent micro-batches)."""
        key = torch.cuda.current_stream(self.device).cuda_stream
        lat, kv = self._expand_bufs.get(key, (None, None))
        if lat is None or lat.numel() < tokens * s.cache_width or kv.numel() < tokens * n:
            latent = [l for l in self.layers if isinstance(l.spec.mixer, LatentSpec)]
            m = max(l.spec.mixer.cache_width for l in latent)
            kn = max(l.mixer.kv.n for l in latent if l.mixer.kv is not None)
            t = pad_to(tokens, 1024)
            lat = torch.empty(t * m, dtype=self.dtype, device=self.device)
            kv = torch.empty(t * kn, dtype=self.dtype, device=self.device)
            self._expand_bufs[key] = (lat, kv)
        return lat[:tokens * s.cache_width].view(tokens, -1), kv[:tokens * n].view(tokens, n)

    def workspace(self, name: str, nbytes: int) -> torch.Tensor:
        """Memory that long portions need (grown on demand: they run eagerly; one per stream of concurrent
        micro-batches)."""
        key = (name, torch.cuda.current_stream(self.device).cuda_stream)
        if key not in self._workspaces or self._workspaces[key].numel() < nbytes:
            self._workspaces[key] = None
            self._workspaces[key] = torch.empty(nbytes, dtype=torch.uint8, device=self.device)
        return self._workspaces[key]

    def rotation(self, s) -> tuple:
        """Tables of a latent attention or a RotarySpec."""
        return self._rot[(s.rot_base, s.rot_dims) if isinstance(s, LatentSpec) else s]

    def memory_bytes(self) -> int:
        ts = [self.embed_w, self.final_norm] + self.k_cache + self.v_cache + [t for s in self.states if s for t in s]
        ts += [t for p in self.pooled for t in p] + (self.loop.tensors() if self.loop is not None else [])
        ts += (self.lm_head.tensors() if self.gpu else [self.lm_head]) if self.has_head else []
        for l in self.layers:
            ts += l.w.tensors()
        seen, n = set(), 0
        for t in ts:
            if t is not None and t.data_ptr() not in seen:
                seen.add(t.data_ptr())
                n += t.numel() * t.element_size()
        return n

    # ------------------------------------------------------------------------- sequences and pages
    @property
    def cache_budget(self) -> int:
        return self.pool.pages

    def cache_need(self, tokens: int) -> int:
        return self.pool.pages_for(tokens)

    def grow(self, slot: int, tokens: int) -> None:
        if self.pool.held[slot] and tokens <= self.max_seq:
            self._ensure(slot, tokens)

    def _ensure(self, slot: int, tokens: int) -> None:
        self.pool.ensure(slot, tokens)
        for p in self.pools.values():
            p.ensure(slot, tokens)

    def reset(self, slots=None) -> None:
        for s in (range(self.max_slots) if slots is None else slots):
            self.seq_len[s] = 0
            for p in (self.pool, *self.pools.values()):
                p.release(s)

    def prefill_rows(self, slot_ids: list, lengths: list) -> tuple:
        out = super().prefill_rows(slot_ids, lengths)
        for s, n in zip(slot_ids, lengths):
            self._ensure(s, self.seq_len[s] + n)
        return out

    # ------------------------------------------------------------------------- forward
    def project(self, lin, x, rows: int, out, glu=None, **kw) -> None:
        lin(x, rows, out, ws=self.coop_ws, sk_ws=self.sk_ws, glu=glu, **kw)

    def project_gated(self, lin, x, rows: int, gate, name: str, key: str) -> dict:
        """stream += sigmoid(gate) * (lin x), in the product's epilogue ({} is left to do); where the stream's
        width does not allow that, what :func:`..ops.stream.stream_join` has to add."""
        W = self.cfg.hidden_size
        if W % 16 == 0:
            self.project(lin, x, rows, None, out32=self.buf_h[:rows], gate=gate, cols=W)
            return {}
        y = self.buf_y[:rows] if name == "y1" else self.scratch_view(name, rows, self.width_p)
        self.project(lin, x, rows, y)
        return {key: (y, gate)} if key == "first" else {key: y, "gate2": gate}

    def embed_into(self, ids: torch.Tensor, h: torch.Tensor) -> None:
        if self.embed_w is None:
            raise RuntimeError("[ERROR] this stage has no embedding layer")
        rows = ids.numel()
        if not self.gpu:
            h.copy_((F.embedding(ids.long(), self.embed_w).float() * self.cfg.embed_scale).repeat(1, self.cfg.streams))
            return
        from ..ops import stream as L
        if self.cfg.streams > 1:
            L.stream_embed(ids, self.embed_w, self.cfg.embed_scale, h, None, rows, self.cfg.streams)
            return
        fits = rows <= self.buf_x.shape[0]
        xc = self.buf_x if fits else torch.empty((rows, self.width_p), dtype=self.dtype, device=self.device)
        L.stream_embed(ids, self.embed_w, self.cfg.embed_scale, h, xc, rows)
        self._x_ready = h.data_ptr() == self.buf_h.data_ptr()  # buf_x holds buf_h's copy

    def embed(self, ids: torch.Tensor) -> torch.Tensor:
        ids = ids.reshape(-1)
        h = torch.empty((ids.numel(), self.cfg.stream_width), dtype=torch.float32, device=self.device)
        self.embed_into(self._i32(ids), h)
        return h

    def forward(self, h: torch.Tensor, slot, pos, kv_len=None) -> torch.Tensor:
        if kv_len is not None:
            raise ValueError("stack engines attend causally (no kv_len)")
        rows = h.shape[0]
        sl, ps = (torch.as_tensor(t, dtype=torch.int64).cpu().reshape(-1) for t in (slot, pos))
        if sl.numel() != rows or ps.numel() != rows or rows < 1:
            raise ValueError("forward: one slot and one position per row")
        if int(sl.min()) < 0 or int(sl.max()) >= self.max_slots or int(ps.min()) < 0 or int(ps.max()) >= self.max_seq:
            raise ValueError("forward: slot or position out of range")
        runs = Plan.find_runs(sl, ps)
        for _, n, s, p in runs:
            self._ensure(s, p + n)
        if not self.gpu:
            return self._forward_stack_torch(h, sl, ps)
        return self._forward_hip(h, self._i32(sl), self._i32(ps), None, rows, runs=runs)

    def latent_nsplit(self, s, entries: int, longest: int) -> int:
        """Key splits of the absorbed attention: about one workgroup per CU (each fills a CU's
        LDS with its two pages), no more splits than pages with visible keys."""
        from ..ops import hip
        from ..ops import latent as L
        if s.window:
            longest = min(longest, s.window + PAGE - 1)  # a window may begin inside a page
        return int(max(1, min(64, hip.N_CU // max(1, entries * L.head_groups(s)), ceil_div(longest, PAGE))))

    def decode_nsplit(self, rows: int) -> int:
        latent = [l.spec.mixer for l in self.layers if isinstance(l.spec.mixer, LatentSpec)]
        return self.latent_nsplit(max(latent, key=lambda m: m.heads), rows, self.max_seq) if latent else 1

    def _forward_hip(self, h, slot, pos, kv_len, rows, nsplit: Optional[int] = None, tiles=None, runs=None):
        from ..ops import stream as L
        if rows > max(self.max_prefill_rows, self.DECODE_MAX_ROWS):
            raise ValueError(f"{rows} rows exceed max_prefill_rows={self.max_prefill_rows}")
        if h.dtype != torch.float32 or not h.is_contiguous():
            h = h.to(torch.float32).contiguous()
        hbuf, x = self.buf_h[:rows], self.buf_x[:rows]
        own = h.data_ptr() == hbuf.data_ptr()
        have = COPY if own and self._x_ready else None
        self._x_ready = False
        if self.loop is not None:
            self.loop.keep(self, h, rows)
        if not own:
            if self.layers[0].w.entry is COPY:
                L.cast_rows(h, x, rows, x2=hbuf)
                have = COPY
            else:
                hbuf.copy_(h)
        if runs is None and nsplit is None:
            nsplit = self.decode_nsplit(rows)
        plan = Plan(self, rows, runs, nsplit)
        ws = [l.w for l in self.layers]
        # what a layer reads: its pass's entry, or its own
        reads = [self.loop if l.spec.enters is not None else l.w.entry for l in self.layers] + [None]
        for i, w in enumerate(ws):
            if reads[i] is self.loop and self.loop is not None:
                have = self.loop.forward(self, rows, self.layers[i].spec.enters, w.entry, have)
            elif have is not w.entry:
                if w.entry is COPY:
                    L.cast_rows(hbuf, x, rows)
                elif isinstance(w.entry, Sum):
                    w.entry.read(self, hbuf, x, rows)
                else:
                    L.stream_norm(hbuf, w.entry, self.cfg.norm_eps, x, rows)
            have = w.forward(self, i, slot, pos, rows, plan, reads[i + 1])
        return hbuf

    def _forward_stack_torch(self, h, slot, pos) -> torch.Tensor:
        x = x0 = h.float()
        for i, l in enumerate(self.layers):
            if l.spec.enters is not None:
                x = self.loop.forward_torch(x, x0, l.spec.enters)
            x = l.w.forward_torch(self, i, x, slot, pos)
        return x

    # ------------------------------------------------------------------------- head
    def _normed(self, h, rows: int, a_rows=None) -> torch.Tensor:
        """Final norm of the selected rows -> the head projection's input."""
        from ..ops import stream as L
        src = h[:rows] if a_rows is None else h.index_select(0, a_rows.long())
        xn = self.buf_x[:rows] if rows <= self.buf_x.shape[0] else torch.zeros(
            (rows, self.width_p), dtype=self.dtype, device=self.device)
        if self.cfg.streams > 1:
            self.head_read.read(self, src, xn, rows)
        else:
            L.stream_norm(src, self.final_norm, self.cfg.norm_eps, xn, rows)
        return xn

    def head_gemv(self, h: torch.Tensor, rows: int, keys: torch.Tensor, a_rows=None) -> None:
        # (a soft cap keeps the order of logits: the largest is the largest before it)
        from ..ops import stream as L
        xn = self._normed(h, rows, a_rows)
        if self.dtype == torch.float32:
            lg = torch.empty((rows, self.lm_head.n), dtype=torch.float32, device=self.device)
            self.lm_head(xn, rows, lg)
            L.logits_argmax(lg, rows, self.head_vocab, keys, offset=self.head_v0)
            return
        self.lm_head(xn, rows, None, ws=self.coop_ws, sk_ws=self.sk_ws, keys=keys, bias=self.head_bias,
                     col_offset=self.head_v0)

    def logits(self, h: torch.Tensor, rows_idx=None) -> torch.Tensor:
        if not self.gpu:
            return super().logits(h, rows_idx)
        from ..ops import stream as L
        idx = None if rows_idx is None else self._i32(rows_idx)
        rows = h.shape[0] if idx is None else idx.numel()
        lg = torch.empty((rows, self.lm_head.n), dtype=torch.float32, device=self.device)
        self.lm_head(self._normed(h, rows, idx), rows, lg, ws=self.coop_ws, sk_ws=self.sk_ws)
        if self.cfg.logit_softcap:
            L.softcap_rows(lg, rows, self.head_vocab, self.cfg.logit_softcap)
        return lg[:, :self.head_vocab]

    def logits_torch(self, hs: torch.Tensor) -> torch.Tensor:
        x = hs.float().view(hs.shape[0], self.cfg.streams, -1).sum(1)
        x = x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + self.cfg.norm_eps) * self.final_norm
        lg = F.linear(x, self.lm_head.float())
        if self.cfg.logit_softcap:
            lg = self.cfg.logit_softcap * torch.tanh(lg / self.cfg.logit_softcap)
        return lg if self.head_bias is None else lg + self.head_bias


__all__ = ["StackEngine"]
