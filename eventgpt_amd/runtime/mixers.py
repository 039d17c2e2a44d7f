"""Token mixers and feed-forwards of the layered decoders: packed weights, per-sequence state, and the
launches that run a batch of rows through them.

Every class takes its declarative spec (``models/layered.py``) and the layer's tensors, packs the weights
for the kernels and owns the state of ``slots`` sequences:

* widths, head sizes and state sizes are padded with zeros to what the kernels' tiles want (``pad``); the
  padding is inert in every product, and norms divide by the true width;
* the projections that read the same input are ONE matrix; the rows that feed fp32 quantities of a recurrence
  (gates, step sizes) come last, so that a long prompt can take them as a separate product with fp32 output
  while everything else is stored in the model's type;
* state is indexed by slot and never cleared: a kernel that sees a sequence's position 0 starts from zeros.

``forward(rows, stream, norm)`` serves both prompts and decode steps; ``rows`` (``RowBatch``) says which.  A prompt
row batch is a pack of sequences without padding between them; a decode batch is one row per slot.  The
residual stream (``Stream``) carries what a sublayer leaves to be added until the next one's norm, so that the
addition, the norm and -- in a decode step of a few sequences -- the next projection are one launch.
"""
from __future__ import annotations

import dataclasses
from typing import Dict, List, Optional, Sequence, Tuple

import torch

from ..models.layered import (AttentionSpec, DenseMLPSpec, LatentAttentionSpec, MatrixMemorySpec, Mamba2Spec, MoESpec,
                              ParallelSpec)

ATTN_TILE = 64           # query rows per work item of the chunk attention
GATE_NONE, GATE_SILU_BEFORE, GATE_SIGMOID_AFTER = 0, 1, 2      # group_norm_rows


def pad(n: int, mult: int) -> int:
    return -(-n // mult) * mult


def pad_value(n: int) -> int:
    """Padded value size of a recurrent head: 32, or a multiple of 64."""
    return 32 if n <= 32 else pad(n, 64)


def pad_attn_head(n: int) -> int:
    """Padded head size of the attention kernels: 64 and 128 have the flash kernels, larger ones the general one."""
    return 64 if n <= 64 else 128 if n <= 128 else pad(n, 64)


def pad_latent(n: int) -> int:
    """Padded latent size: 64, or a multiple of 128."""
    return 64 if n <= 64 else pad(n, 128)


def pad_rows(w: torch.Tensor, groups: int, size: int, padded: int) -> torch.Tensor:
    """``[groups * size, ...] -> [groups * padded, ...]`` with zero rows after each group."""
    rest = w.shape[1:]
    out = w.new_zeros(groups, padded, *rest)
    out[:, :size] = w.reshape(groups, size, *rest)
    return out.reshape(groups * padded, *rest)


def pad_cols(w: torch.Tensor, groups: int, size: int, padded: int) -> torch.Tensor:
    return pad_rows(w.t().contiguous(), groups, size, padded).t().contiguous()


def pad_to(w: torch.Tensor, *shape: int) -> torch.Tensor:
    out = w.new_zeros(*shape)
    out[tuple(slice(n) for n in w.shape)] = w
    return out


@dataclasses.dataclass
class Sequence_:
    slot: int
    row0: int        # first row in the pack
    rows: int
    start: int       # position of the first row


class RowBatch:
    """Rows of one pass.  ``decode``: row ``b`` is the next token of slot ``b`` at the device position ``pos[b]``.
    Otherwise a pack of sequence portions, with the index tables the kernels read, built once per pass and
    shared by all layers."""

    def __init__(self, device, decode: bool, pos: Optional[torch.Tensor] = None, live: Optional[torch.Tensor] = None,
                 seqs: Sequence[Sequence_] = (), scan_chunk: int = 64):
        """``scan_chunk``: tokens per chunk of the recurrences' prefill kernels (``raw.scan_chunk``)."""
        self.device, self.decode, self.live = device, decode, live
        self.seqs: List[Sequence_] = list(seqs)
        self._tables: Dict = {}
        if decode:
            self.pos, self.slot, self.first = pos, None, None
            return
        slot, ps, first, chunks, seq_rows, tails = [], [], [], [], [], []
        for s in self.seqs:
            slot += [s.slot] * s.rows
            ps += range(s.start, s.start + s.rows)
            first += [s.row0] * s.rows
            n = -(-s.rows // scan_chunk)
            end = (s.start + s.rows) & 1
            seq_rows += [len(chunks) // 4, n, s.slot, int(s.start == 0) | (s.start & 1) << 1 | end << 2]
            for c in range(n):
                chunks += [s.row0 + c * scan_chunk, min(scan_chunk, s.rows - c * scan_chunk), s.slot,
                           int(c == n - 1) | end << 1]
            tails += [s.row0, s.rows, s.slot, s.start]
        self.slot, self.pos, self.first, self.chunks, self.scan_seqs, self.tails = self._upload(
            slot, ps, first, chunks, seq_rows, tails)
        self.chunks, self.scan_seqs, self.tails = (t.view(-1, 4) for t in (self.chunks, self.scan_seqs, self.tails))

    def _upload(self, *lists):
        """Several int lists in one copy to the device."""
        flat = torch.tensor([v for l in lists for v in l], dtype=torch.int32).to(self.device)
        return flat.split([len(l) for l in lists])

    def chunk_tables(self, size: int):
        """For a chunk mask of ``size``: ``(runs, items, row_kv, row_keep, copies, kv_rows)``.  Keys live in a buffer
        with the rows of every sequence in order, preceded by the cached keys of the chunk it continues."""
        t = self._tables.get(size)
        if t is not None:
            return t
        runs: List[Tuple[int, int, int, int, int]] = []     # q row, rows, key row of the chunk, position in it, repeats
        items: List[int] = []
        row_kv: List[int] = []
        keep: List[int] = []
        copies: List[int] = []
        kv = 0
        for s in self.seqs:
            pre = s.start % size
            if pre:
                copies += [s.slot, 0, kv, pre]
            base = kv + pre
            row_kv += range(base, base + s.rows)
            live_from = (s.start + s.rows) // size * size    # the chunk the next token belongs to
            keep += [int(p >= live_from) for p in range(s.start, s.start + s.rows)]
            done = 0
            while done < s.rows:
                off = (s.start + done) % size
                n = min(size - off, s.rows - done)
                reps = (s.rows - done) // size if off == 0 and n == size else 1
                key0 = base + done - off
                runs.append((s.row0 + done, n, key0, off, reps))
                for r in range(reps):
                    for a in range(0, n, ATTN_TILE):
                        items += [s.row0 + done + r * n + a, min(ATTN_TILE, n - a), key0 + r * n, off + a]
                done += n * reps
            kv = base + s.rows
        items_d, row_kv_d, keep_d, copies_d = self._upload(items, row_kv, keep, copies)
        t = (runs, items_d.view(-1, 4), row_kv_d, keep_d, copies_d.view(-1, 4) if copies else None, kv)
        self._tables[size] = t
        return t

    def causal_tables(self):
        """For plain causal attention: ``(runs, items, copies, kv_rows)`` of ``chunk_tables``, where a buffer holds
        every key of every sequence and ``copies`` brings all of them from the caches."""
        t = self._tables.get("causal")
        if t is None:
            runs: List[Tuple[int, int, int, int, int]] = []
            items: List[int] = []
            copies: List[int] = []
            kv = 0
            for s in self.seqs:
                runs.append((s.row0, s.rows, kv, s.start, 1))
                for a in range(0, s.rows, ATTN_TILE):
                    items += [s.row0 + a, min(ATTN_TILE, s.rows - a), kv, s.start + a]
                copies += [s.slot, 0, kv, s.start + s.rows]
                kv += s.start + s.rows
            items_d, copies_d = self._upload(items, copies)
            t = self._tables["causal"] = (runs, items_d.view(-1, 4), copies_d.view(-1, 4), kv)
        return t

    def latents(self, cache: torch.Tensor, gather) -> torch.Tensor:
        """All cached rows of the pack's sequences, in the order of ``causal_tables``; shared by the layers that read
        this cache.  ``gather(cache, copies, rows)`` copies them where they are not already one run of the cache."""
        key = ("latents", cache.data_ptr())
        t = self._tables.get(key)
        if t is None:
            _, _, copies, kv = self.causal_tables()
            one = self.seqs[0]
            t = cache[one.slot, :kv] if len(self.seqs) == 1 else gather(cache, copies, kv)
            self._tables[key] = t
        return t


class Stream:
    """The fp32 residual rows, with the last sublayer's contribution possibly still to be added.  ``pending`` is None or
    names how: ``("add", y)`` the rows or slabs ``y``; ``("merge", a, b, wa, wb)`` the mean of two normed branches;
    ``("post", y, w)`` the normed ``y``; ``("mix", y, pick, weights, w)`` the weighted sum of picked rows of ``y``, normed
    if there is a ``w``.  ``post`` is the weight of the norm after the current sublayer, or None."""

    def __init__(self, engine, x: torch.Tensor, decode: bool):
        self.raw, self.n, self.eps, self.f32 = engine.raw, engine.width, engine.eps, engine.dtype == torch.float32
        self.layer = engine.layer_norm
        self.x, self.pending, self.post = x, None, None
        self.few = decode and x.shape[0] <= engine.gemv_rows

    def leave(self, y: torch.Tensor) -> None:
        """The current sublayer's output, to be added."""
        self.pending = ("add", y) if self.post is None else ("post", y, self.post)

    def normed(self, norm: Optional[torch.Tensor]) -> torch.Tensor:
        """Norm of the stream in the storage type, pending contribution included (None: just add it)."""
        pending, self.pending = self.pending, None
        last = (norm, self.n, self.eps, self.f32)
        if pending is None:
            return self.raw.norm_rows(self.x, None, *last, self.layer) if norm is not None else None
        kind, *args = pending
        if kind == "add":
            return self.raw.add_norm_rows_(self.x, *args, *last, self.layer)
        if kind == "post":
            return self.raw.post_norm_rows_(self.x, *args, *last, self.layer)
        if kind == "mix":
            return self.raw.mix_norm_rows_(self.x, *args, *last, self.layer)
        return self.raw.merge_norm_rows_(self.x, *args, *last)

    def settle(self) -> torch.Tensor:
        if self.pending is not None:
            self.normed(None)
        return self.x

    def gemv(self, norm: torch.Tensor, w: torch.Tensor, act: int = -1, xn: Optional[torch.Tensor] = None,
             scale: Optional[float] = None, cap: float = 0.0) -> torch.Tensor:
        """``w`` times the normed stream in one launch (a few rows): fp32 rows, or ``act(gate) * up``.  ``xn`` also gets the
        normed rows; ``scale`` and ``cap``: the rows are ``cap tanh(scale y / cap)``."""
        pending, self.pending = self.pending, None
        if pending is not None and pending[0] in ("add", "mix"):
            self.pending = pending
            self.settle()
            pending = None
        last = (self.layer, xn, scale, cap)
        if pending is None:
            return self.raw.gemv_norm(self.x, norm, self.n, self.eps, w, act, None, None, None, None, None, *last)
        out = torch.empty_like(self.x)       # blocks read the old stream while one of them writes the new one
        kind, *args = pending
        a, b, wa, wb = args if kind == "merge" else (args[0], None, args[1], None)
        y = self.raw.gemv_norm(self.x, norm, self.n, self.eps, w, act, a, b, wa, wb, out, *last)
        self.x = out
        return y


class Projection:
    """Row-stacked projections of one input: sections in the model's type, then the fp32 gate rows."""

    def __init__(self, raw, sections: List[Tuple[str, torch.Tensor]], gates: List[Tuple[str, torch.Tensor]], k_pad: int):
        self.raw, self.col = raw, {}
        n, parts = 0, []
        for name, w in sections:
            self.col[name] = n
            n += w.shape[0]
            parts.append(w)
        if n % 8:
            raise ValueError("projection sections must be multiples of eight rows")
        g = 0
        for name, w in gates:
            self.col[name] = n + g           # column in a decode step's rows; a prompt has the gates on their own
            g += w.shape[0]
            parts.append(w)
        self.n_main = n
        self.w = pad_to(torch.cat(parts), n + pad(g, 8), k_pad)
        self.w_main, self.w_gate = self.w[:n], self.w[n:]

    def step(self, stream: Stream, norm: torch.Tensor) -> torch.Tensor:
        """All sections as fp32 rows ``[B, N]`` or slabs ``[S, B, N]``."""
        if stream.few:
            return stream.gemv(norm, self.w)
        return self.raw.linear_slabs(stream.normed(norm), self.w)

    def prompt(self, stream: Stream, norm: torch.Tensor):
        """``(sections in the storage type, gate sections in fp32)``."""
        xn = stream.normed(norm)
        return self.raw.linear(xn, self.w_main, False), self.raw.linear(xn, self.w_gate, True) if self.w_gate.shape[0] else None

    def gate_col(self, name: str) -> int:
        return self.col[name] - self.n_main


class Mixer:
    def __init__(self, engine):
        """``engine``: widths, dtype, slots, rotation tables."""
        self.raw, self.eps = engine.raw, engine.eps
        self.dtype, self.f32 = engine.dtype, engine.dtype == torch.float32
        self.width, self.wp, self.device, self.slots = engine.width, engine.wp, engine.device, engine.B
        self._lds = engine.gemv_lds // (4 if self.f32 else 2)      # elements of input rows a GEMV block can hold

    def _w32(self, t: torch.Tensor) -> torch.Tensor:
        return t.float().contiguous()

    def few(self, stream: Stream, k: int) -> bool:
        """A few rows, and inputs of ``k`` elements (plus per-head factors) fit the GEMV's LDS."""
        return stream.few and stream.x.shape[0] * k + 4096 <= self._lds


class AttentionBranch(Mixer):
    def __init__(self, engine, spec: AttentionSpec, t):
        """``t(name)``: the layer's tensor of that name."""
        super().__init__(engine)
        self.spec = spec
        self.D = D = pad_attn_head(max(spec.dim, spec.vdim))
        if D > 512:
            raise ValueError(f"attention heads of {max(spec.dim, spec.vdim)} elements (at most 512)")
        self.size = min(spec.chunk or engine.l_max, engine.l_max)
        H, G = spec.heads, spec.kv_heads
        self.sections = [("lq", pad_rows(t("q"), H, spec.dim, D)), ("lk", pad_rows(t("k"), G, spec.dim, D)),
                         ("lv", pad_rows(t("v"), G, spec.vdim, D))]
        self.qw = self._w32(pad_rows(t("q.norm"), H, spec.dim, D))
        self.kw = self._w32(pad_rows(t("k.norm"), G, spec.dim, D))
        self.w_o = pad_to(pad_cols(t("o"), H, spec.vdim, D), self.wp, pad(H * D, 64))
        self.cos, self.sin = engine.rotation(spec.rot_base, spec.rot_dims)
        shape = (self.slots, G, self.size, D)
        self.k_cache = torch.zeros(shape, dtype=self.dtype, device=self.device)
        self.v_cache = torch.zeros(shape, dtype=self.dtype, device=self.device)
        self.nsplit = engine.kv_splits(self.slots, H)

    def dims(self, col: Dict[str, int]) -> List[int]:
        s = self.spec
        return [col["lq"], col["lk"], col["lv"], s.heads, s.kv_heads, self.D, s.heads * s.dim, s.kv_heads * s.dim]

    def step(self, rows: RowBatch, q: torch.Tensor) -> torch.Tensor:
        o = self.raw.attn_chunk_decode(q, self.k_cache, self.v_cache, rows.pos, self.spec.scale, self.nsplit)
        return o.view(o.shape[0], -1)

    def prompt(self, rows: RowBatch, src: torch.Tensor, col: Dict[str, int]) -> torch.Tensor:
        s, raw = self.spec, self.raw
        runs, items, row_kv, keep, copies, kv_rows = rows.chunk_tables(self.size)
        k = torch.empty(kv_rows, s.kv_heads, self.D, dtype=self.dtype, device=self.device)
        v = torch.empty_like(k)
        if copies is not None:      # before the cache slots of the chunk are written over
            raw.chunk_keys_copy_(self.k_cache, self.v_cache, k, v, copies)
        lq, lk, lv, H, G, D, nq, nk = self.dims(col)
        q = raw.attn_prep_(src, lq, lk, lv, self.qw, self.kw, H, G, D, nq, nk, self.eps, self.cos, self.sin, rows.slot,
                           rows.pos, row_kv, keep, k, v, self.k_cache, self.v_cache)
        # few long runs: the flash kernel, one launch each; many short ones: one launch for all
        if not self.f32 and D <= 128 and len(runs) <= 4 * len(rows.seqs) and max(r[1] for r in runs) > 256:
            o = torch.empty_like(q)
            for q0, n, key0, off, reps in runs:
                raw.attn_runs_(q, k, v, o, q0, n, key0, off, reps, s.scale)
        else:
            o = raw.attn_chunk(q, k, v, items, s.scale)
        return o.view(o.shape[0], -1)


class MatrixMemoryBranch(Mixer):
    def __init__(self, engine, spec: MatrixMemorySpec, t):
        super().__init__(engine)
        self.spec = spec
        self.N, self.V = N, V = pad(spec.dim, 32), pad_value(spec.vdim)
        H = spec.heads
        self.sections = [("rq", pad_rows(t("q"), H, spec.dim, N)), ("rk", pad_rows(t("k"), H, spec.dim, N)),
                         ("rv", pad_rows(t("v"), H, spec.vdim, V)), ("rg", pad_rows(t("g"), H, spec.vdim, V))]
        self.gates = [("ri", t("i")), ("rf", t("f"))]
        self.ib, self.fb = self._w32(t("i.b")), self._w32(t("f.b"))
        self.norm = self._w32(pad_rows(t("norm"), H, spec.vdim, V))
        self.kp = pad(H * V, 64)
        self.w_o = pad_to(pad_cols(t("o"), H, spec.vdim, V), self.wp, self.kp)
        self.qscale = spec.dim ** -0.5
        f = dict(dtype=torch.float32, device=self.device)
        self.S = torch.zeros(self.slots, H, V, N, **f)
        # normaliser and running maximum, two images each: indexed by the parity of the position that reads them
        self.n = torch.zeros(2, self.slots, H, N, **f)
        self.m = torch.zeros(2, self.slots, H, **f)

    def dims(self, col: Dict[str, int]) -> List[int]:
        return [col["rq"], col["rk"], col["rv"], col["ri"], col["rf"], self.spec.heads, self.N, self.V]

    def gated(self, o: torch.Tensor, src: torch.Tensor, col: Dict[str, int]) -> torch.Tensor:
        """Per-head norm and output gate."""
        H = self.spec.heads
        return self.raw.group_norm_rows(o, src, col["rg"], GATE_SIGMOID_AFTER, self.norm, H, self.spec.vdim, self.V, H,
                                        self.kp, self.eps, self.f32)

    def prompt(self, rows: RowBatch, src: torch.Tensor, gates: torch.Tensor, proj: Projection) -> torch.Tensor:
        raw, H, N, V, c = self.raw, self.spec.heads, self.N, self.V, proj.col
        li, lf = raw.mlstm_gates(gates, proj.gate_col("ri"), proj.gate_col("rf"), self.ib, self.fb, self.spec.gate_cap)
        q, k, v = src[:, c["rq"]:c["rk"]], src[:, c["rk"]:c["rv"]], src[:, c["rv"]:c["rg"]]
        o = raw.scan_prefill_(q, k, v, H, 1, N, V, self.qscale, lf, li, None, None, self.S, self.n, self.m, rows.chunks,
                              rows.scan_seqs)
        return self.gated(o, src, c)


class ParallelMixer(Mixer):
    """Two mixers on the same input; their outputs are left to the residual kernel that norms and averages them."""

    def __init__(self, engine, spec: ParallelSpec, t):
        super().__init__(engine)
        self.left = AttentionBranch(engine, spec.left, lambda n: t("left." + n))
        self.right = MatrixMemoryBranch(engine, spec.right, lambda n: t("right." + n))
        self.proj = Projection(engine.raw, self.left.sections + self.right.sections, self.right.gates, self.wp)
        self.left.sections = self.right.sections = self.right.gates = None
        self.w_left = pad_to(self._w32(t("left.out")), self.wp)
        self.w_right = pad_to(self._w32(t("right.out")), self.wp)

    def forward(self, rows: RowBatch, stream: Stream, norm: torch.Tensor) -> None:
        raw, left, right, col = self.raw, self.left, self.right, self.proj.col
        if rows.decode:
            src = self.proj.step(stream, norm)
            q, mem = raw.parallel_step_(src, left.dims(col), left.qw, left.kw, self.eps, left.cos, left.sin, left.k_cache,
                                        left.v_cache, right.dims(col), right.ib, right.fb, right.spec.gate_cap, right.qscale,
                                        right.S, right.n, right.m, rows.pos, rows.live)
            o = left.step(rows, q)
            if self.few(stream, max(left.w_o.shape[1], right.kp)):
                a, b = raw.gemv_branches(left.w_o, o, right.w_o, mem, src, col["rg"], right.norm, right.spec.heads,
                                         right.spec.vdim, right.V, self.eps).unbind(0)
            else:
                a = raw.linear_slabs(o, left.w_o)
                b = raw.linear_slabs(right.gated(mem, src, col), right.w_o)
        else:
            src, gates = self.proj.prompt(stream, norm)
            a = raw.linear(left.prompt(rows, src, col), left.w_o, True)
            b = raw.linear(right.prompt(rows, src, gates, self.proj), right.w_o, True)
        stream.pending = ("merge", a, b, self.w_left, self.w_right)


class Mamba2Mixer(Mixer):
    def __init__(self, engine, spec: Mamba2Spec, t):
        super().__init__(engine)
        self.spec = s = spec
        self.N, self.V = N, V = pad(s.state, 32), pad_value(s.vdim)
        H, G = s.heads, s.groups
        z, x, b, c, dt = t("in").split([s.inner, s.inner, G * s.state, G * s.state, H])
        self.proj = Projection(engine.raw, [("z", pad_rows(z, H, s.vdim, V)), ("x", pad_rows(x, H, s.vdim, V)),
                                            ("b", pad_rows(b, G, s.state, N)), ("c", pad_rows(c, G, s.state, N))],
                               [("dt", dt)], self.wp)

        def channels(w):
            x, b, c = w.split([s.inner, G * s.state, G * s.state])
            return self._w32(torch.cat([pad_rows(x, H, s.vdim, V), pad_rows(b, G, s.state, N), pad_rows(c, G, s.state, N)]))
        self.conv_w, self.conv_b = channels(t("conv")), channels(t("conv.b"))
        self.dt_bias, self.a_log, self.skip = (self._w32(t(n)) for n in ("dt_bias", "A_log", "D"))
        self.norm = self._w32(pad_rows(t("norm"), H, s.vdim, V))
        self.kp = pad(H * V, 64)
        self.w_o = pad_to(pad_cols(t("o"), H, s.vdim, V), self.wp, self.kp)
        self.ring = torch.zeros(self.slots, s.conv, self.conv_w.shape[0], dtype=self.dtype, device=self.device)
        self.S = torch.zeros(self.slots, H, V, N, dtype=torch.float32, device=self.device)

    def forward(self, rows: RowBatch, stream: Stream, norm: torch.Tensor) -> None:
        s, raw, H, G, N, V, col = self.spec, self.raw, self.spec.heads, self.spec.groups, self.N, self.V, self.proj.col
        head_norm = (self.norm, H, s.vdim, V, s.norm_groups)
        if rows.decode:
            src = self.proj.step(stream, norm)
            y = raw.ssd_step_(src, [col["z"], col["x"], col["dt"], H, G, N, V], self.conv_w, self.conv_b, self.ring,
                              self.dt_bias, self.a_log, self.skip, self.S, rows.pos, rows.live)
            if self.few(stream, self.kp) and stream.post is None:
                raw.gemv_group_add_(stream.settle(), self.w_o, y, *head_norm, self.eps)
                return
            y = raw.group_norm_rows(y, None, 0, GATE_NONE, *head_norm, self.kp, self.eps, self.f32)
            stream.leave(raw.linear_slabs(y, self.w_o))
            return
        src, gates = self.proj.prompt(stream, norm)
        log_decay, dt = raw.ssd_gates(gates, self.proj.gate_col("dt"), self.dt_bias, self.a_log)
        xbc = raw.conv_rows_(src, col["x"], self.conv_w, self.conv_b, self.ring, rows.slot, rows.pos, rows.first)
        raw.conv_tail_(src, col["x"], self.ring, rows.tails)
        xs, b, c = xbc[:, :H * V], xbc[:, H * V:H * V + G * N], xbc[:, H * V + G * N:]
        y = raw.scan_prefill_(c, b, xs, H, H // G, N, V, 1.0, log_decay, None, dt, self.skip, self.S, None, None, rows.chunks,
                              rows.scan_seqs)
        y = raw.group_norm_rows(y, src, col["z"], GATE_SILU_BEFORE, *head_norm, self.kp, self.eps, self.f32)
        stream.leave(raw.linear(y, self.w_o, True))


class LatentAttentionMixer(Mixer):
    """A prompt expands the latents of its keys to keys and values of every head and runs the causal attention kernels on
    them; a decode step (and a short portion of a long sequence) takes its queries into the latent space instead and
    attends over the cached rows themselves."""

    def __init__(self, engine, spec: LatentAttentionSpec, t):
        super().__init__(engine)
        self.spec = s = spec
        self.D = D = pad_attn_head(max(s.dim, s.vdim))
        self.R = R = pad_latent(s.kv_rank)
        self.Q = Q = pad(s.q_rank, 64)
        if D > 512 or R > self.raw.latent_max():
            raise ValueError(f"heads of {max(s.dim, s.vdim)} and latents of {s.kv_rank} elements (at most 512, {self.raw.latent_max()})")
        H = s.heads
        sections = [("q", pad_to(t("dq"), Q, self.width))]
        self.cache = None
        if s.kv_from is None:
            sections.append(("c", pad_to(t("dkv"), R, self.width)))
            self.c_norm = pad_to(self._w32(t("dkv.norm")), R)
            self.cache = torch.zeros(self.slots, engine.l_max, R, dtype=self.dtype, device=self.device)
        sections.append(("g", pad_to(t("g"), pad(H, 8), self.width)))
        self.owner = self if s.kv_from is None else engine.mixers[s.kv_from]
        self.proj = Projection(engine.raw, sections, [], self.wp)
        self.q_norm = pad_to(self._w32(t("dq.norm")), Q)
        self.w_uq = pad_to(pad_rows(t("uq"), H, s.dim, D), H * D, Q)
        uk, uv = pad_to(pad_rows(t("uk"), H, s.dim, D), H * D, R), pad_to(pad_rows(t("uv"), H, s.vdim, D), H * D, R)
        self.w_ukv = torch.cat([uk, uv])                                   # a prompt's keys and values
        self.w_absorb = uk.view(H, D, R).transpose(1, 2).contiguous()      # queries into the latent space [H, R, D]
        self.w_value = self.w_ukv[H * D:].view(H, D, R)                    # attended latents out of it
        self.w_o = pad_to(pad_cols(t("o"), H, s.vdim, D), self.wp, H * D)

    def splits(self, rows: int) -> int:
        """Key splits of the attention over the cache: about one workgroup per CU."""
        tiles = -(-self.spec.heads // 32)
        return max(1, min(64, 256 // max(1, rows * tiles)))

    def absorbs(self, rows: RowBatch) -> bool:
        """Whether a pack's queries attend over the cached rows: few of them per key, so that expanding every key costs
        more.  (Work per head in multiply-adds; a quarter of the rate of the prompt kernels.)"""
        if any(s.start == 0 for s in rows.seqs):
            return False
        R, D, expand, direct = self.R, self.D, 0, 0
        for s in rows.seqs:
            keys = s.start + s.rows
            expand += 2 * keys * D * (R + s.rows)
            direct += 2 * s.rows * (keys * R * 4 + D * R)
        return direct < expand

    def attend(self, rows: RowBatch, q: torch.Tensor, src: torch.Tensor) -> torch.Tensor:
        """Gated attention outputs of query rows ``[M, H * D]``, over the cache."""
        raw, s = self.raw, self.spec
        ql = raw.head_linear(q, self.w_absorb, None, 0)
        o = raw.latent_attend(ql, self.owner.cache, rows.slot, rows.pos, s.scale, self.splits(ql.shape[0]), self.w_value, src,
                              self.proj.col["g"])
        return o.view(o.shape[0], -1)

    def prompt_attention(self, rows: RowBatch, q: torch.Tensor, src: torch.Tensor) -> torch.Tensor:
        raw, s, D = self.raw, self.spec, self.D
        H = s.heads
        runs, items, _, kv_rows = rows.causal_tables()
        kv = raw.linear(rows.latents(self.owner.cache, raw.latent_gather), self.w_ukv, False)
        q, k, v = q.view(-1, H, D), kv[:, :H * D].unflatten(1, (H, D)), kv[:, H * D:].unflatten(1, (H, D))
        gate = (src, self.proj.col["g"])
        if not self.f32 and D <= 128 and max(r[1] for r in runs) > 256:
            o = torch.empty_like(q)
            for q0, n, key0, off, reps in runs:
                raw.attn_runs_(q, k, v, o, q0, n, key0, off, reps, s.scale, *gate)
        else:
            o = raw.attn_chunk(q, k, v, items, s.scale, *gate)
        return o.view(o.shape[0], -1)

    def forward(self, rows: RowBatch, stream: Stream, norm: torch.Tensor) -> None:
        raw, s, col = self.raw, self.spec, self.proj.col
        store = (col["c"], s.kv_rank, self.c_norm, self.cache) if self.cache is not None else (0, 0, None, None)
        src = self.proj.step(stream, norm) if rows.decode else self.proj.prompt(stream, norm)[0]
        if rows.decode and self.few(stream, self.Q):
            q = raw.gemv_rows(src, col["q"], s.q_rank, self.q_norm, self.eps, self.w_uq, *store, rows.pos, rows.live)
        else:
            cq = raw.latent_prep_(src, col["q"], s.q_rank, self.q_norm, *store, rows.slot, rows.pos, rows.live, self.eps, self.f32)
            q = raw.linear_slabs(cq, self.w_uq) if rows.decode else raw.linear(cq, self.w_uq, False)
        if rows.decode or self.absorbs(rows):
            o = self.attend(rows, q, src)
        else:
            o = self.prompt_attention(rows, q, src)
        stream.leave(raw.gemv_plain(self.w_o, o) if stream.few else
                     raw.linear_slabs(o, self.w_o) if rows.decode else raw.linear(o, self.w_o, True))


class DenseMLP(Mixer):
    def __init__(self, engine, spec: DenseMLPSpec, t):
        super().__init__(engine)
        from ..ops.layered import GLU_ACTS
        self.act = GLU_ACTS[spec.act]
        fp = pad(spec.ff, 64)
        self.w_gate_up = torch.cat([pad_to(t("gate"), fp, self.wp), pad_to(t("up"), fp, self.wp)])
        self.w_down = pad_to(t("down"), self.wp, fp)

    def forward(self, rows: RowBatch, stream: Stream, norm: torch.Tensor) -> None:
        raw = self.raw
        if stream.few:
            h = stream.gemv(norm, self.w_gate_up, self.act)
            if stream.post is None:
                raw.gemv_add_(stream.settle(), self.w_down, h)
            else:
                stream.leave(raw.gemv_plain(self.w_down, h))
            return
        h = raw.linear_glu(stream.normed(norm), self.w_gate_up, self.act)
        stream.leave(raw.linear_slabs(h, self.w_down) if rows.decode else raw.linear(h, self.w_down, True))


class MoE(Mixer):
    """Mixture of experts.  A few rows stream the weights of their own experts; more rows are sorted by expert and go through
    grouped products, and the residual kernel sums each row's share of them."""

    def __init__(self, engine, spec: MoESpec, t):
        super().__init__(engine)
        from ..ops.layered import GLU_ACTS
        self.spec, self.act = spec, GLU_ACTS[spec.act]
        fp, E = pad(spec.ff, 64), spec.experts
        self.w_router = pad_to(t("router"), pad(E, 8), self.wp)
        self.bias = self._w32(t("router.b"))
        self.w_gate_up = torch.stack([torch.cat([pad_to(t(f"e{e}.gate"), fp, self.wp), pad_to(t(f"e{e}.up"), fp, self.wp)])
                                      for e in range(E)])
        self.w_down = torch.stack([pad_to(t(f"e{e}.down"), self.wp, fp) for e in range(E)])

    def forward(self, rows: RowBatch, stream: Stream, norm: torch.Tensor) -> None:
        raw, top = self.raw, self.spec.top
        if stream.few:
            xn = torch.empty(stream.x.shape, dtype=self.dtype, device=self.device)
            logits = stream.gemv(norm, self.w_router, xn=xn)
            y = raw.moe_step(xn, logits, self.bias, top, self.w_gate_up, self.w_down, self.act)
            stream.leave(y)
            return
        xn = stream.normed(norm)
        logits = raw.linear_slabs(xn, self.w_router)
        idx, weights = raw.moe_route(logits, self.bias, top)
        perm, inv, start = raw.moe_group(idx, self.spec.experts)
        h = raw.moe_linear(xn, self.w_gate_up, start, perm, top, self.act)
        y = raw.moe_linear(h, self.w_down, start, None, 1, -1)
        stream.pending = ("mix", y, inv, weights, stream.post)


MIXERS = {"parallel": ParallelMixer, "mamba2": Mamba2Mixer, "latent_attention": LatentAttentionMixer}
MLPS = {DenseMLPSpec: DenseMLP, MoESpec: MoE}
