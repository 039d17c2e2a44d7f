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

from ..models.layered import AttentionSpec, DenseMLPSpec, MatrixMemorySpec, Mamba2Spec, ParallelSpec

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


class Stream:
    """The fp32 residual rows, with the last sublayer's contribution possibly still to be added: ``pending`` is None,
    ``(y,)`` (add the rows or slabs ``y``) or ``(a, b, wa, wb)`` (add the mean of the two normed branches)."""

    def __init__(self, engine, x: torch.Tensor, decode: bool):
        self.raw, self.n, self.eps, self.f32 = engine.raw, engine.width, engine.eps, engine.dtype == torch.float32
        self.x, self.pending = x, None
        self.few = decode and x.shape[0] <= engine.gemv_rows

    def normed(self, norm: Optional[torch.Tensor]) -> torch.Tensor:
        """RMS norm of the stream in the storage type, pending contribution included (None: just add it)."""
        pending, self.pending = self.pending, None
        if pending is None:
            return self.raw.norm_rows(self.x, None, norm, self.n, self.eps, self.f32) if norm is not None else None
        if len(pending) == 1:
            return self.raw.add_norm_rows_(self.x, pending[0], norm, self.n, self.eps, self.f32)
        return self.raw.merge_norm_rows_(self.x, *pending, norm, self.n, self.eps, self.f32)

    def settle(self) -> torch.Tensor:
        if self.pending is not None:
            self.normed(None)
        return self.x

    def gemv(self, norm: torch.Tensor, w: torch.Tensor, act: int = -1) -> torch.Tensor:
        """``w`` times the normed stream in one launch (a few rows): fp32 rows, or ``act(gate) * up``."""
        pending, self.pending = self.pending, None
        if pending is not None and len(pending) == 1:
            self.pending = pending
            self.settle()
            pending = None
        if pending is None:
            return self.raw.gemv_norm(self.x, norm, self.n, self.eps, w, act, None, None, None, None, None)
        out = torch.empty_like(self.x)       # blocks read the old stream while one of them writes the new one
        y = self.raw.gemv_norm(self.x, norm, self.n, self.eps, w, act, *pending, out)
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
        return self.raw.linear(xn, self.w_main, False), self.raw.linear(xn, self.w_gate, True)

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
        stream.pending = (a, b, self.w_left, self.w_right)


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
            if self.few(stream, self.kp):
                raw.gemv_group_add_(stream.settle(), self.w_o, y, *head_norm, self.eps)
                return
            y = raw.group_norm_rows(y, None, 0, GATE_NONE, *head_norm, self.kp, self.eps, self.f32)
            stream.pending = (raw.linear_slabs(y, self.w_o),)
            return
        src, gates = self.proj.prompt(stream, norm)
        log_decay, dt = raw.ssd_gates(gates, self.proj.gate_col("dt"), self.dt_bias, self.a_log)
        xbc = raw.conv_rows_(src, col["x"], self.conv_w, self.conv_b, self.ring, rows.slot, rows.pos, rows.first)
        raw.conv_tail_(src, col["x"], self.ring, rows.tails)
        xs, b, c = xbc[:, :H * V], xbc[:, H * V:H * V + G * N], xbc[:, H * V + G * N:]
        y = raw.scan_prefill_(c, b, xs, H, H // G, N, V, 1.0, log_decay, None, dt, self.skip, self.S, None, None, rows.chunks,
                              rows.scan_seqs)
        y = raw.group_norm_rows(y, src, col["z"], GATE_SILU_BEFORE, *head_norm, self.kp, self.eps, self.f32)
        stream.pending = (raw.linear(y, self.w_o, True),)


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
            raw.gemv_add_(stream.settle(), self.w_down, h)
            return
        h = raw.linear_glu(stream.normed(norm), self.w_gate_up, self.act)
        stream.pending = (raw.linear_slabs(h, self.w_down) if rows.decode else raw.linear(h, self.w_down, True),)


MIXERS = {"parallel": ParallelMixer, "mamba2": Mamba2Mixer}
