"""Layered text decoders: a stack whose layers each name their token mixer and its sizes.

``config.json`` lists the layers in order; every entry gives a ``type``, that mixer's own sizes
(``mixer``) and a feed-forward (``mlp``, or null).  The classes here are the declarative half: they read
the configuration, say which tensors a checkpoint of it holds, and keep those tensors.  What a mixer
computes, how its weights are packed and what it keeps per sequence is ``runtime/mixers.py``; the serving
path is ``runtime/layered_engine.LayeredEngine``.

Designs built from these parts:

* **Nusitar** -- layers of type ``parallel`` (a chunk-masked softmax attention and an mLSTM matrix memory
  side by side on the same input) and ``mamba2`` (state-space duality with a short convolution), an fp32
  residual stream, gelu-gated feed-forwards.
"""
from __future__ import annotations

import copy
import dataclasses
import json
import os
from typing import Any, Dict, List, Optional, Tuple

import torch

from ..utils.checkpoint import load_into, save_sharded

Shapes = Dict[str, Tuple[int, ...]]


def _take(d: Dict[str, Any], where: str, *names: str, **optional):
    """The named values of a configuration object; anything it holds besides them is refused, so a
    configuration that asks for a mechanism this code does not have cannot be half understood."""
    unknown = set(d) - set(names) - set(optional)
    missing = [n for n in names if n not in d]
    if unknown or missing:
        raise ValueError(f"{where}: missing {missing}, unknown {sorted(unknown)}")
    return tuple(d[n] for n in names) + tuple(d.get(n, v) for n, v in optional.items())


def _positive(where: str, **sizes) -> None:
    for n, v in sizes.items():
        if not isinstance(v, int) or v < 1:
            raise ValueError(f"{where}.{n} must be a positive integer, got {v!r}")


@dataclasses.dataclass(frozen=True)
class AttentionSpec:
    """Softmax attention with grouped key / value heads, an RMS norm over the whole q and k projections,
    partial rotary positions and a chunk mask (``chunk`` None: plain causal)."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_dims: int
    rot_base: float
    chunk: Optional[int]

    @classmethod
    def from_dict(cls, d, where) -> "AttentionSpec":
        heads, kv, dim, vdim, scale, rot, mask = _take(d, where, "heads", "kv_heads", "dim", "vdim", "scale", "rot", "mask")
        dims, base = _take(rot, where + ".rot", "dims", "base")
        size = None if mask is None else _take(mask, where + ".mask", "size")[0]
        _positive(where, heads=heads, kv_heads=kv, dim=dim, vdim=vdim)
        if heads % kv or dims < 0 or dims % 2 or dims > dim:
            raise ValueError(f"{where}: {heads} heads over {kv} key heads, {dims} of {dim} dimensions rotated")
        if size is not None:
            _positive(where + ".mask", size=size)
        return cls(heads, kv, dim, vdim, float(scale), dims, float(base), size)

    def shapes(self, p: str, width: int) -> Shapes:
        q, k, v = self.heads * self.dim, self.kv_heads * self.dim, self.kv_heads * self.vdim
        return {p + "q": (q, width), p + "k": (k, width), p + "v": (v, width), p + "q.norm": (q,), p + "k.norm": (k,),
                p + "o": (width, self.heads * self.vdim)}


@dataclasses.dataclass(frozen=True)
class MatrixMemorySpec:
    """mLSTM: a matrix state per head with exponential input gate, sigmoid forget gate, running maximum."""
    heads: int
    dim: int
    vdim: int
    gate_cap: float

    @classmethod
    def from_dict(cls, d, where) -> "MatrixMemorySpec":
        heads, dim, vdim, cap = _take(d, where, "heads", "dim", "vdim", "gate_cap")
        _positive(where, heads=heads, dim=dim, vdim=vdim)
        if not cap > 0:
            raise ValueError(f"{where}.gate_cap must be positive")
        return cls(heads, dim, vdim, float(cap))

    def shapes(self, p: str, width: int) -> Shapes:
        qk, v, h = self.heads * self.dim, self.heads * self.vdim, self.heads
        return {p + "q": (qk, width), p + "k": (qk, width), p + "v": (v, width), p + "g": (v, width), p + "o": (width, v),
                p + "norm": (v,), p + "i": (h, width), p + "i.b": (h,), p + "f": (h, width), p + "f.b": (h,)}


@dataclasses.dataclass(frozen=True)
class ParallelSpec:
    """Attention and matrix memory on the same input; their outputs are normed and averaged."""
    left: AttentionSpec
    right: MatrixMemorySpec

    @classmethod
    def from_dict(cls, d, where) -> "ParallelSpec":
        left, right = _take(d, where, "left", "right")
        return cls(AttentionSpec.from_dict(left, where + ".left"), MatrixMemorySpec.from_dict(right, where + ".right"))

    def shapes(self, p: str, width: int) -> Shapes:
        return {**self.left.shapes(p + "left.", width), **self.right.shapes(p + "right.", width),
                p + "left.out": (width,), p + "right.out": (width,)}


@dataclasses.dataclass(frozen=True)
class Mamba2Spec:
    heads: int
    groups: int
    state: int
    vdim: int
    conv: int
    norm_groups: int

    @classmethod
    def from_dict(cls, d, where) -> "Mamba2Spec":
        spec = cls(*_take(d, where, "heads", "groups", "state", "vdim", "conv", "norm_groups"))
        _positive(where, **dataclasses.asdict(spec))
        if spec.heads % spec.groups or spec.inner % spec.norm_groups:
            raise ValueError(f"{where}: heads over groups, or inner size over norm_groups, does not divide")
        return spec

    @property
    def inner(self) -> int:
        return self.heads * self.vdim

    @property
    def channels(self) -> int:
        return self.inner + 2 * self.groups * self.state

    def shapes(self, p: str, width: int) -> Shapes:
        h = self.heads
        return {p + "in": (self.inner + self.channels + h, width), p + "conv": (self.channels, self.conv),
                p + "conv.b": (self.channels,), p + "dt_bias": (h,), p + "A_log": (h,), p + "D": (h,),
                p + "norm": (self.inner,), p + "o": (width, self.inner)}


@dataclasses.dataclass(frozen=True)
class DenseMLPSpec:
    """``W_down(gelu_tanh(W_gate h) * W_up h)``."""
    ff: int
    act: str = "gelu_tanh"

    @classmethod
    def from_dict(cls, d, where) -> "DenseMLPSpec":
        kind, ff = _take(d, where, "kind", "ff")
        if kind != "dense":
            raise ValueError(f"{where}.kind {kind!r} is not supported")
        _positive(where, ff=ff)
        return cls(ff)

    def shapes(self, p: str, width: int) -> Shapes:
        return {p + "gate": (self.ff, width), p + "up": (self.ff, width), p + "down": (width, self.ff)}


MIXER_SPECS = {"parallel": ParallelSpec, "mamba2": Mamba2Spec}


@dataclasses.dataclass(frozen=True)
class LayerSpec:
    type: str
    mixer: Any
    mlp: Optional[DenseMLPSpec]

    def shapes(self, p: str, width: int) -> Shapes:
        out = {p + "norm1": (width,), **self.mixer.shapes(p + "mix.", width)}
        if self.mlp is not None:
            out[p + "norm2"] = (width,)
            out.update(self.mlp.shapes(p + "mlp.", width))
        return out


class LayeredConfig:
    """Configuration of a layered decoder (``architecture``, ``vocab``, ``width``, ``norm.eps``,
    ``embedding.scale`` and the list of ``layers``)."""

    def __init__(self, d: Dict[str, Any]):
        self.raw = copy.deepcopy(d)
        known = ("architecture", "vocab", "width", "norm", "embedding", "layers")
        arch, vocab, width, norm, emb, layers = _take({k: d[k] for k in known if k in d}, "config", *known)
        self.architecture = arch
        _positive("config", vocab=vocab, width=width)
        self.vocab_size, self.hidden_size = vocab, width
        self.norm_eps = float(_take(norm, "norm", "eps")[0])
        self.embedding_scale = float(_take(emb, "embedding", "scale")[0])
        self.eos_token_id = d.get("eos_token_id")
        self.layers: List[LayerSpec] = []
        for i, e in enumerate(layers):
            kind, mixer, mlp = _take(e, f"layers[{i}]", "type", "mixer", "mlp")
            if kind not in MIXER_SPECS:
                raise ValueError(f"layers[{i}].type {kind!r}: known are {sorted(MIXER_SPECS)}")
            self.layers.append(LayerSpec(kind, MIXER_SPECS[kind].from_dict(mixer, f"layers[{i}].mixer"),
                                         None if mlp is None else DenseMLPSpec.from_dict(mlp, f"layers[{i}].mlp")))
        if not self.layers:
            raise ValueError("config: no layers")

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "LayeredConfig":
        return cls(d)

    @classmethod
    def from_pretrained(cls, path: str) -> "LayeredConfig":
        with open(os.path.join(path, "config.json")) as f:
            return cls(json.load(f))

    def to_dict(self) -> Dict[str, Any]:
        return copy.deepcopy(self.raw)

    def save_pretrained(self, path: str) -> None:
        os.makedirs(path, exist_ok=True)
        with open(os.path.join(path, "config.json"), "w") as f:
            json.dump(self.raw, f, indent=1, sort_keys=True)

    def parameter_shapes(self) -> Shapes:
        out: Shapes = {"embed": (self.vocab_size, self.hidden_size)}
        for i, layer in enumerate(self.layers):
            out.update(layer.shapes(f"l{i}.", self.hidden_size))
        out["final.norm"] = (self.hidden_size,)
        out["head"] = (self.vocab_size, self.hidden_size)
        return out


class LayeredDecoder:
    """A configuration and its tensors.  Inference runs on ``engine()`` (GPU); ``generate`` is the entry
    point the command line uses."""

    def __init__(self, config: LayeredConfig, dtype: torch.dtype = torch.bfloat16, device="cpu"):
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"dtype {dtype}: bfloat16 or float32")
        self.config, self.dtype, self.device = config, dtype, torch.device(device)
        self.tensors = {n: torch.empty(s, dtype=dtype, device=self.device) for n, s in config.parameter_shapes().items()}
        self._engine = None

    def state_dict(self, keep_vars: bool = False) -> Dict[str, torch.Tensor]:
        return self.tensors

    # ------------------------------------------------------------ construction
    @classmethod
    def from_pretrained(cls, path: str, torch_dtype: torch.dtype = torch.bfloat16, config: Optional[LayeredConfig] = None,
                        device="cpu") -> "LayeredDecoder":
        model = cls(config or LayeredConfig.from_pretrained(path), torch_dtype, device)
        load_into(model, path, strict=True, ignore_suffixes=(), grown_vocab=False)
        return model

    @classmethod
    def from_config(cls, config: LayeredConfig, torch_dtype: torch.dtype = torch.bfloat16, device="cpu",
                    seed: int = 0) -> "LayeredDecoder":
        """Random weights: matrices scaled by fan-in, norms near one, decays spread over a few decades."""
        model = cls(config, torch_dtype, device)
        g = torch.Generator(device=model.device).manual_seed(seed)
        for name, t in model.tensors.items():
            z = torch.randn(t.shape, generator=g, device=t.device, dtype=torch.float32)
            leaf = name.rsplit(".", 1)[-1]
            if leaf.startswith("norm") or leaf == "out" or leaf == "D":
                z = 1 + 0.1 * z
            elif leaf == "A_log":
                z = 0.5 * z
            elif leaf == "dt_bias":
                z = z - 2
            elif name.endswith(".f.b"):
                z = z + 3
            elif name.endswith(".i.b"):
                z = z - 3
            elif t.dim() == 2:
                z = z / t.shape[1] ** 0.5
            t.copy_(z)
        return model

    def save_pretrained(self, path: str) -> None:
        self.config.save_pretrained(path)
        save_sharded(self.tensors, path)

    # ----------------------------------------------------------------- serving
    def eval(self) -> "LayeredDecoder":
        return self

    def engine(self, max_len: int = 4096, max_batch: int = 1, **kw):
        """The serving engine; an existing one is reused while it is large enough."""
        from ..runtime.layered_engine import LayeredEngine
        e = self._engine
        if e is None or e.l_max < max_len or e.B < max_batch:
            self._engine = None
            self._engine = e = LayeredEngine(self, max_len=max_len, max_batch=max_batch, **kw)
        return e

    def generate(self, input_ids: torch.Tensor, do_sample: bool = False, temperature: float = 1.0, top_p: float = 1.0,
                 top_k: int = 0, max_new_tokens: int = 512, eos_token_id: Optional[int] = None,
                 generator: Optional[torch.Generator] = None, **_) -> torch.Tensor:
        """New token ids ``[1, n]`` after the prompt ``input_ids [1, S]`` (or ``[S]``)."""
        ids = input_ids.reshape(-1)
        eos = eos_token_id if eos_token_id is not None else self.config.eos_token_id
        e = self.engine(max_len=max(4096, ids.numel() + max_new_tokens), max_new_tokens=max(1024, max_new_tokens))
        if e.max_out < max_new_tokens:
            self._engine = None
            e = self.engine(max_len=e.l_max, max_new_tokens=max_new_tokens)
        out = e.generate(ids, max_new_tokens, temperature if do_sample else 0.0, top_p, -1 if eos is None else eos,
                         generator, top_k)
        return out[None]
