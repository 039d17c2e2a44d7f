"""LayeredEngine -- the serving path of the layered decoders (``models/layered.LayeredDecoder``).

It is a ``DecodeEngine``: positions, token rings, EOS flags, graph capture, generation, sampling and slot
scheduling are the ones the other models use, and ``runtime.batcher.ContinuousBatcher`` drives it.  What
it adds is the stack of mixers (``runtime/mixers.py``) over an fp32 residual stream:

* a prompt is token ids; several prompts prefill as one pack without padding, long ones in portions;
* what a sequence keeps depends on the layer -- the current chunk's keys, a recurrent state, the last inputs
  of a convolution, a latent per token (which several layers may read) -- and is held per slot in static
  buffers, so a decode step is one captured graph;
* ``active`` masks a slot's state updates as well as its commit: a recurrent state, unlike a cache row, may
  not be written twice for the same token.

Weights, activations and caches are bf16 or, for a float32 model, fp32 throughout.
"""
from __future__ import annotations

from typing import Dict, List, Optional, Sequence, Tuple

import torch

from .engine import DecodeEngine, GenerationEngine, persistent_state
from .mixers import MIXERS, MLPS, RowBatch, Sequence_, Stream, pad, pad_to


class _Stage:
    """One residual sublayer, the norm weights that lead into it and those of the norm after it (or None)."""

    def __init__(self, block, norm, post):
        self.block, self.norm, self.post = block, norm, post


class LayeredEngine(DecodeEngine):
    #: most rows one prefill pass carries; longer prompts run in portions of it
    PACK_ROWS = 8192

    kv_splits = staticmethod(GenerationEngine.kv_splits)

    @persistent_state
    def __init__(self, model, max_len: int = 4096, max_batch: int = 1, use_graph: bool = True,
                 max_new_tokens: int = 1024, poll_every: int = 16):
        from ..ops import layered            # raises if the extension is missing
        self.raw = layered.raw
        cfg = model.config
        if model.device.type != "cuda":
            raise RuntimeError("LayeredEngine needs the model on a GPU")
        self.model, self.cfg, self.device, self.dtype = model, cfg, model.device, model.dtype
        self.B, self.l_max, self.max_out = max_batch, max_len, max_new_tokens
        self.use_graph, self.poll_every = use_graph, poll_every
        self.f32 = self.dtype == torch.float32
        self.width, self.wp, self.eps = cfg.hidden_size, pad(cfg.hidden_size, 64), cfg.norm_eps
        self.V = cfg.vocab_size
        self.layer_norm = cfg.design.norm == "layer"
        # logits = cap tanh(scale * logits / cap), or None
        self._finish = None if cfg.logit_scale == 1.0 and cfg.logit_softcap is None else (cfg.logit_scale, cfg.logit_softcap or 0.0)
        # decode steps of up to this many sequences run on the weight-streaming kernels, more on the few-row GEMM
        self.gemv_rows = int(self.raw.gemv_rows_max())
        self.scan_chunk = int(self.raw.scan_chunk(self.f32))
        self.gemv_lds = int(self.raw.gemv_lds_bytes())
        if self.wp * (4 if self.f32 else 2) * min(self.B, self.gemv_rows) > self.gemv_lds:
            self.gemv_rows = 0
        self._rot: Dict[Tuple[float, int], Tuple[torch.Tensor, torch.Tensor]] = {}
        t = model.tensors

        def norm(name):
            return pad_to(t[name].float(), self.wp)
        self.embed = pad_to(t["embed"], self.V, self.wp)
        self.head = pad_to(t["head"], pad(self.V, 8), self.wp)
        self.final_norm = norm("final.norm")
        self.stages: List[_Stage] = []
        self.layer_ends: List[int] = []      # number of stages after each layer
        self.mixers: List = []               # one per layer; a layer may read an earlier one's cache
        for i, layer in enumerate(cfg.layers):
            p = f"l{i}."

            def post(n):
                return norm(p + n) if layer.post_norm else None
            self.mixers.append(MIXERS[layer.type](self, layer.mixer, lambda n: t[p + "mix." + n]))
            self.stages.append(_Stage(self.mixers[-1], norm(p + "norm1"), post("norm1b")))
            if layer.mlp is not None:
                block = MLPS[type(layer.mlp)](self, layer.mlp, lambda n: t[p + "mlp." + n])
                self.stages.append(_Stage(block, norm(p + "norm2"), post("norm2b")))
            self.layer_ends.append(len(self.stages))
        self._init_decode_state(torch.zeros(self.B, self.wp, dtype=torch.float32, device=self.device), cfg.eos_token_id)
        self.active = torch.ones(self.B, dtype=torch.int32, device=self.device)
        self._fed = [0] * self.B             # tokens given to each slot through ``extend``

    def rotation(self, base: float, dims: int):
        """``cos, sin [max_len, dims / 2]`` of the rotary angles, fp32 (angles in double)."""
        key = (base, dims)
        if key not in self._rot:
            half = dims // 2
            f = base ** (-2.0 * torch.arange(half, dtype=torch.float64, device=self.device) / max(dims, 1))
            a = torch.arange(self.l_max, dtype=torch.float64, device=self.device)[:, None] * f
            self._rot[key] = (a.cos().float().contiguous(), a.sin().float().contiguous())
        return self._rot[key]

    # ------------------------------------------------------------------ layers
    def _run_stages(self, rows: RowBatch, x: torch.Tensor, collect: Optional[list] = None) -> Stream:
        """All layers over the residual rows ``x`` (updated in place, or replaced in the stream that is returned)."""
        stream = Stream(self, x, rows.decode)
        for i, st in enumerate(self.stages):
            stream.post = st.post
            st.block.forward(rows, stream, st.norm)
            if collect is not None and i + 1 in self.layer_ends:
                collect.append(stream.settle()[:, :self.width].clone())
        return stream

    def _logits(self, xn: torch.Tensor) -> torch.Tensor:
        logits = self.raw.linear(xn, self.head, True)
        if self._finish:
            self.raw.cap_logits_(logits, *self._finish)
        return logits[:, :self.V]

    def _layers_step(self) -> None:
        rows = RowBatch(self.device, True, pos=self.pos, live=self.active)
        self._stream = self._run_stages(rows, self.x)

    def _logits_and_commit(self, greedy: bool, want_logits: bool = False) -> None:
        stream, self._stream = self._stream, None
        if stream is None:                   # after a prefill: ``x`` holds the last rows' residual stream
            stream = Stream(self, self.x, True)
        if stream.few:
            logits = stream.gemv(self.final_norm, self.head, -1, None, *(self._finish or (None, 0.0)))[:, :self.V]
        else:
            logits = self._logits(stream.normed(self.final_norm))
        if not greedy or want_logits:
            self.logits.copy_(logits)
        if greedy:
            self._commit(logits)

    _stream: Optional[Stream] = None

    def _commit_sampled(self) -> None:
        self._commit(None)

    def _commit(self, logits: Optional[torch.Tensor]) -> None:
        """Commit ``sampled``, or the argmax of ``logits``, and stage the next token's embedding."""
        self.raw.commit_rows_(logits, self.sampled, self.embed, self.cfg.embedding_scale, self.x, self.out_tokens, self.step,
                              self.pos, self.done, self.cur_token, self.eos, self.active)

    def _capture(self, fn):
        """The warm-up run of a capture must not advance any sequence's state."""
        saved = self.active.clone()
        self.active.zero_()
        try:
            return super()._capture(fn)
        finally:
            self.active.copy_(saved)

    def reset(self) -> None:
        super().reset()
        self.active.fill_(1)
        self._fed = [0] * self.B

    # ----------------------------------------------------------------- prefill
    def _pack(self, slots: Sequence[int], ids: Sequence[torch.Tensor], starts: Sequence[int],
              collect: Optional[list] = None) -> Tuple[torch.Tensor, List[int]]:
        """One pass over portions ``ids[i]`` of the sequences in ``slots``, from position ``starts[i]`` on:
        ``(residual rows, first row of each portion)``."""
        seqs, n = [], 0
        for slot, t, start in zip(slots, ids, starts):
            if start + t.numel() > self.l_max:
                raise ValueError(f"sequence of {start + t.numel()} tokens exceeds max_len ({self.l_max})")
            seqs.append(Sequence_(int(slot), n, int(t.numel()), int(start)))
            n += int(t.numel())
        flat = torch.cat([t.reshape(-1).to("cpu", torch.int32) if not t.is_cuda else t.reshape(-1).to(torch.int32) for t in ids])
        x = self.raw.embed_rows(flat.to(self.device).contiguous(), self.embed, self.cfg.embedding_scale)
        stream = self._run_stages(RowBatch(self.device, False, seqs=seqs, scan_chunk=self.scan_chunk), x, collect)
        return stream.settle(), [s.row0 for s in seqs]

    def _packs(self, slots, ids, starts):
        """Cut portions into passes of at most ``PACK_ROWS`` rows: ``[(slots, ids, starts, indices, offsets)]``."""
        out, cur, room = [], None, 0
        for i, (slot, t, start) in enumerate(zip(slots, ids, starts)):
            off, n = 0, int(t.numel())
            while off < n:
                # a sequence's next portion needs the state its last one leaves: never two in one pass
                if cur is None or room == 0 or i in cur[3]:
                    cur, room = ([], [], [], [], []), self.PACK_ROWS
                    out.append(cur)
                take = min(room, n - off)
                for lst, v in zip(cur, (slot, t[off:off + take], start + off, i, off)):
                    lst.append(v)
                off += take
                room -= take
        return out

    @torch.no_grad()
    def _feed(self, slots, ids, starts, want=None):
        """Append ``ids[i]`` to the sequences; returns the last residual row of each and the logits at the
        wanted places (``want[i]``: places in ``ids[i]``) in order."""
        ids = [t.reshape(-1) for t in ids]
        if any(t.numel() == 0 for t in ids):
            raise ValueError("an empty prompt has no last token to continue from")
        last: List[Optional[torch.Tensor]] = [None] * len(ids)
        rows: Dict[Tuple[int, int], torch.Tensor] = {}
        for p_slots, p_ids, p_starts, idx, offs in self._packs(slots, ids, starts):
            x, row0 = self._pack(p_slots, p_ids, p_starts)
            sel, keys = [], []
            for i, off, t, r in zip(idx, offs, p_ids, row0):
                if off + t.numel() == ids[i].numel():
                    last[i] = x[r + t.numel() - 1].clone()
                for w in (want[i] if want is not None else ()):
                    if off <= w < off + t.numel():
                        sel.append(r + w - off)
                        keys.append((i, w))
            if sel:
                picked = torch.tensor(sel, dtype=torch.int32).to(self.device)
                lg = self._logits(self.raw.norm_rows(x, picked, self.final_norm, self.width, self.eps, self.f32,
                                                       self.layer_norm))
                rows.update(zip(keys, lg))
        logits = None
        if want is not None and any(len(w) for w in want):
            logits = torch.stack([rows[(i, w)] for i, ws in enumerate(want) for w in ws])
        return last, logits

    def _prefill_slots(self, slots: Sequence[int], prompts: Sequence[torch.Tensor]) -> None:
        last, _ = self._feed(slots, prompts, [0] * len(slots))
        for b, t, row in zip(slots, prompts, last):
            self.x[b].copy_(row)
            self.pos[b] = t.numel() - 1          # the commit advances it to the prompt length
            self._pos_hi = max(self._pos_hi, int(t.numel()))

    @torch.no_grad()
    def prefill(self, ids: torch.Tensor, batch: int = 0, start: Optional[int] = None, select: Optional[str] = "greedy"):
        """Run token ids through the decoder, appending to sequence ``batch`` from position ``start`` (default: its
        current length).  ``select`` as in ``GenerationEngine.prefill``."""
        ids = ids.reshape(-1)
        if start is None:
            start = int(self.pos[batch].item())
        last, _ = self._feed([batch], [ids], [start])
        self._pos_hi = max(self._pos_hi, start + ids.numel())
        self._fed[batch] = start + ids.numel()
        if select is None:
            self.pos[batch] = start + ids.numel()
            return
        self.pos[batch] = start + ids.numel() - 1
        self.x[batch].copy_(last[0])
        self._logits_and_commit(greedy=(select == "greedy"))

    # ------------------------------------------------------------ given tokens
    @torch.no_grad()
    def extend(self, slots: Sequence[int], tokens: Sequence[torch.Tensor], want: Sequence[Sequence[int]]):
        """Feed given tokens (nothing is sampled): ``tokens[i]`` continues the sequence in ``slots[i]``.  Single
        tokens of running sequences go through the decode step, everything else through the packed prefill.
        Returns the logits ``[n, V]`` at the wanted places, in order, or None."""
        starts = [self._fed[s] for s in slots]
        step = all(t.numel() == 1 and s > 0 for t, s in zip(tokens, starts))
        for s, t in zip(slots, tokens):
            self._fed[s] += int(t.numel())
        if not step:
            _, logits = self._feed(slots, tokens, starts, want)
            for s in slots:
                self.pos[s] = self._fed[s] - 1
            self._pos_hi = max([self._pos_hi] + [self._fed[s] for s in slots])
            return logits
        if max(self._fed) > self.l_max:
            raise ValueError(f"sequence exceeds max_len ({self.l_max})")
        self.active.zero_()
        self.active[list(slots)] = 1
        self.sampled[list(slots)] = torch.cat([t.reshape(-1) for t in tokens]).to(self.device, torch.int32)
        self._commit_sampled()
        self.decode_step(greedy=False)
        rows = [s for s, w in zip(slots, want) for _ in w]
        return self.logits[rows].clone() if rows else None

    def release(self, slots: Sequence[int]) -> None:
        """Give the slots of finished sequences back."""
        self.park(slots)
        self.step[list(slots)] = 0
        for s in slots:
            self._fed[s] = 0

    def layer_outputs(self, ids: torch.Tensor) -> torch.Tensor:
        """Residual stream after every layer of one prompt, ``[layers, S, width]`` fp32 (slot 0 is overwritten)."""
        out: list = []
        self._pack([0], [ids.reshape(-1)], [0], out)
        return torch.stack(out)
