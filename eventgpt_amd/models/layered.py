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
* **Zapipel** -- layers of type ``latent_attention`` (one cached latent per token, which layers can share),
  layer norms before and after every sublayer, silu-gated feed-forwards that are dense or a mixture of
  experts, logits scaled and softly capped.
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
class LatentAttentionSpec:
    """Softmax attention whose keys and values are linear in one RMS-normed latent per token, the only thing
    that is cached.  Queries go through a latent of their own; every head has a sigmoid output gate; there are no
    positions.  ``kv_from``: the layer whose latents this one reads instead of having its own."""
    heads: int
    dim: int
    vdim: int
    kv_rank: int
    q_rank: int
    scale: float
    kv_from: Optional[int] = None

    @classmethod
    def from_dict(cls, d, where) -> "LatentAttentionSpec":
        heads, dim, vdim, kv_rank, q_rank, scale, src = _take(d, where, "heads", "dim", "vdim", "kv_rank", "q_rank", "scale",
                                                              kv_from=None)
        _positive(where, heads=heads, dim=dim, vdim=vdim, kv_rank=kv_rank, q_rank=q_rank)
        if not scale > 0:
            raise ValueError(f"{where}.scale must be positive")
        return cls(heads, dim, vdim, kv_rank, q_rank, float(scale), src)

    def check(self, index: int, earlier: List["LayerSpec"], where: str) -> None:
        """``kv_from`` names an earlier layer with latents of its own and of this size."""
        j = self.kv_from
        if j is None:
            return
        if not isinstance(j, int) or not 0 <= j < index:
            raise ValueError(f"{where}.kv_from {j!r} is not an earlier layer")
        other = earlier[j].mixer
        if not isinstance(other, LatentAttentionSpec) or other.kv_from is not None or other.kv_rank != self.kv_rank:
            raise ValueError(f"{where}.kv_from: layer {j} has no latents of its own of size {self.kv_rank}")

    def shapes(self, p: str, width: int) -> Shapes:
        h = self.heads
        out = {p + "dq": (self.q_rank, width), p + "dq.norm": (self.q_rank,), p + "uq": (h * self.dim, self.q_rank),
               p + "uk": (h * self.dim, self.kv_rank), p + "uv": (h * self.vdim, self.kv_rank), p + "g": (h, width),
               p + "o": (width, h * self.vdim)}
        if self.kv_from is None:
            out.update({p + "dkv": (self.kv_rank, width), p + "dkv.norm": (self.kv_rank,)})
        return out


@dataclasses.dataclass(frozen=True)
class DenseMLPSpec:
    """``W_down(act(W_gate h) * W_up h)``."""
    ff: int
    act: str

    @classmethod
    def from_dict(cls, d, where, act) -> "DenseMLPSpec":
        _, ff = _take(d, where, "kind", "ff")
        _positive(where, ff=ff)
        return cls(ff, act)

    def shapes(self, p: str, width: int) -> Shapes:
        return {p + "gate": (self.ff, width), p + "up": (self.ff, width), p + "down": (width, self.ff)}


@dataclasses.dataclass(frozen=True)
class MoESpec:
    """Mixture of ``experts`` gated units of ``ff``: a token uses the ``top`` ones with the largest router logits,
    weighted by the softmax over those logits."""
    experts: int
    top: int
    ff: int
    act: str

    @classmethod
    def from_dict(cls, d, where, act) -> "MoESpec":
        _, expert, router = _take(d, where, "kind", "expert", "router")
        (ff,) = _take(expert, where + ".expert", "ff")
        experts, top = _take(router, where + ".router", "experts", "top")
        _positive(where, ff=ff, experts=experts, top=top)
        if top > experts:
            raise ValueError(f"{where}.router: {top} of {experts} experts")
        return cls(experts, top, ff, act)

    def shapes(self, p: str, width: int) -> Shapes:
        out = {p + "router": (self.experts, width), p + "router.b": (self.experts,)}
        for i in range(self.experts):
            out.update(DenseMLPSpec(self.ff, self.act).shapes(f"{p}e{i}.", width))
        return out


MIXER_SPECS = {"parallel": ParallelSpec, "mamba2": Mamba2Spec, "latent_attention": LatentAttentionSpec}
MLP_SPECS = {"dense": DenseMLPSpec, "moe": MoESpec}


@dataclasses.dataclass(frozen=True)
class Design:
    """What an architecture fixes: its layer types and feed-forwards, the gated units' activation, the kind of norm and
    where it stands, and the keys its configuration has besides the common ones."""
    mixers: Tuple[str, ...]
    mlps: Tuple[str, ...]
    act: str
    norm: str = "rms"              # "rms" or "layer"
    post_norm: bool = False        # a norm of every sublayer's output as well
    keys: Tuple[str, ...] = ()


DESIGNS = {
    "Nusitar": Design(("parallel", "mamba2"), ("dense",), "gelu_tanh", keys=("embedding",)),
    "Zapipel": Design(("latent_attention",), ("dense", "moe"), "silu", norm="layer", post_norm=True,
                      keys=("logit_scale", "logit_softcap")),
}


@dataclasses.dataclass(frozen=True)
class LayerSpec:
    type: str
    mixer: Any
    mlp: Any                       # DenseMLPSpec, MoESpec or None
    post_norm: bool = False

    def shapes(self, p: str, width: int) -> Shapes:
        out = {p + "norm1": (width,), **self.mixer.shapes(p + "mix.", width)}
        if self.post_norm:
            out[p + "norm1b"] = (width,)
        if self.mlp is not None:
            out[p + "norm2"] = (width,)
            if self.post_norm:
                out[p + "norm2b"] = (width,)
            out.update(self.mlp.shapes(p + "mlp.", width))
        return out


class LayeredConfig:
    """Configuration of a layered decoder: ``architecture``, ``vocab``, ``width``, ``norm.eps``, the list of ``layers``
    and what the architecture has besides (``embedding.scale``; ``logit_scale``, ``logit_softcap``)."""

    def __init__(self, d: Dict[str, Any]):
        self.raw = copy.deepcopy(d)
        arch = d.get("architecture")
        if arch not in DESIGNS:
            raise ValueError(f"architecture {arch!r}: known are {sorted(DESIGNS)}")
        self.architecture, self.design = arch, DESIGNS[arch]
        known = ("vocab", "width", "norm", "layers") + self.design.keys
        vocab, width, norm, layers, *_ = _take({k: d[k] for k in known if k in d}, "config", *known)
        _positive("config", vocab=vocab, width=width)
        self.vocab_size, self.hidden_size = vocab, width
        self.norm_eps = float(_take(norm, "norm", "eps")[0])
        has = self.design.keys
        self.embedding_scale = float(_take(d["embedding"], "embedding", "scale")[0]) if "embedding" in has else 1.0
        self.logit_scale = float(d["logit_scale"]) if "logit_scale" in has else 1.0
        #: logits are ``cap * tanh(logits / cap)``; None: they are not capped
        cap = d["logit_softcap"] if "logit_softcap" in has else None
        if cap is not None and not cap > 0:
            raise ValueError("config.logit_softcap must be positive")
        self.logit_softcap = None if cap is None else float(cap)
        self.eos_token_id = d.get("eos_token_id")
        self.layers: List[LayerSpec] = []
        for i, e in enumerate(layers):
            kind, mixer, mlp = _take(e, f"layers[{i}]", "type", "mixer", "mlp")
            if kind not in self.design.mixers:
                raise ValueError(f"layers[{i}].type {kind!r}: {arch} has {sorted(self.design.mixers)}")
            spec = MIXER_SPECS[kind].from_dict(mixer, f"layers[{i}].mixer")
            if isinstance(spec, LatentAttentionSpec):
                spec.check(i, self.layers, f"layers[{i}].mixer")
            if mlp is not None and mlp.get("kind") not in self.design.mlps:
                raise ValueError(f"layers[{i}].mlp.kind {mlp.get('kind')!r}: {arch} has {sorted(self.design.mlps)}")
            ff = None if mlp is None else MLP_SPECS[mlp["kind"]].from_dict(mlp, f"layers[{i}].mlp", self.design.act)
            self.layers.append(LayerSpec(kind, spec, ff, self.design.post_norm))
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
            elif name.endswith("router.b"):
                z = 0.1 * z
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
