"""Prefill and decode throughput of a layered decoder beside a LLaMA decoder of equal size.

``bench.py --layered 1b,7b [--layered-design nusitar|zapipel]`` runs this; weights are random, layers have the
sizes of real models of that width, the stack is ``2 n`` layers (Nusitar: ``mamba2``, ``parallel``, ...;
Zapipel: latent attention with a dense feed-forward, then on the same latents with experts, ...) and the LLaMA
stack has the number of layers that comes closest in the parameters a token uses.  Every row prints both models'
time and what it means against the bound of that pass: decoder weights over time for decode steps, 2 x parameters
x tokens over time for prompts.
"""
from __future__ import annotations

import json
import re
import time
from typing import Dict, List

import torch

SIZES: Dict[str, Dict[str, int]] = {
    "1b": dict(width=2048, ff=5632, heads=16, kv_heads=4, memory_heads=4, mamba_heads=64, groups=4, q_rank=768, expert_ff=2816),
    "7b": dict(width=4096, ff=11008, heads=32, kv_heads=8, memory_heads=8, mamba_heads=128, groups=8, q_rank=1536, expert_ff=5504),
}
KV_RANK, EXPERTS, TOP = 512, 8, 2


def layered_config(size: str, pairs: int, vocab: int = 32000) -> dict:
    s = SIZES[size]
    rec = {"heads": s["memory_heads"], "dim": 256, "vdim": 512, "gate_cap": 15.0}
    att = {"heads": s["heads"], "kv_heads": s["kv_heads"], "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
           "rot": {"dims": 128, "base": 10000.0}, "mask": {"size": 2048}}
    par = {"type": "parallel", "mixer": {"left": att, "right": rec}, "mlp": {"kind": "dense", "ff": s["ff"]}}
    mam = {"type": "mamba2", "mlp": None, "mixer": {"heads": s["mamba_heads"], "groups": s["groups"], "state": 128,
                                                    "vdim": 64, "conv": 4, "norm_groups": s["groups"]}}
    return {"architecture": "Nusitar", "vocab": vocab, "width": s["width"], "norm": {"eps": 1e-6},
            "embedding": {"scale": 1.0}, "layers": [mam, par] * pairs}


def latent_config(size: str, pairs: int, vocab: int = 32000) -> dict:
    s = SIZES[size]
    mix = {"heads": s["heads"], "dim": 128, "vdim": 128, "kv_rank": KV_RANK, "q_rank": s["q_rank"], "scale": 128 ** -0.5}
    layers = []
    for i in range(pairs):
        layers.append({"type": "latent_attention", "mixer": mix, "mlp": {"kind": "dense", "ff": s["ff"]}})
        layers.append({"type": "latent_attention", "mixer": {**mix, "kv_from": 2 * i},
                       "mlp": {"kind": "moe", "expert": {"ff": s["expert_ff"]}, "router": {"experts": EXPERTS, "top": TOP}}})
    return {"architecture": "Zapipel", "vocab": vocab, "width": s["width"], "norm": {"eps": 1e-6}, "logit_scale": 1.0,
            "logit_softcap": 30.0, "layers": layers}


CONFIGS = {"nusitar": layered_config, "zapipel": latent_config}


def layer_params(model) -> int:
    """Matrix parameters of the decoder layers that a token uses (no embedding, no head; the chosen experts)."""
    named = model.tensors.items() if hasattr(model, "tensors") else ((n, p) for n, p in model.model.named_parameters())
    skip = ("embed", "head", "visual", "feature")
    return sum(t.numel() * (TOP / EXPERTS if re.search(r"mlp\.e\d+\.", n) else 1)
               for n, t in named if t.dim() == 2 and not any(k in n for k in skip))


def llama_like(size: str, params: int, vocab: int, dev):
    from ..models import ClipVisionConfig, EventChatConfig, EventChatModel
    s = SIZES[size]
    per = 4 * s["width"] ** 2 + 3 * s["width"] * s["ff"]
    cfg = EventChatConfig(vocab_size=vocab, hidden_size=s["width"], intermediate_size=s["ff"],
                          num_hidden_layers=max(1, round(params / per)), num_attention_heads=s["heads"],
                          max_position_embeddings=16384, mm_visual_tower="small", event_feature_adaptor=True)
    cfg.vision_config = ClipVisionConfig(hidden_size=64, intermediate_size=128, num_hidden_layers=1, num_attention_heads=2,
                                         image_size=28, patch_size=14)
    return EventChatModel.from_config(cfg, torch.bfloat16, dev, seed=0)


def _time(fn, n: int) -> float:
    """Best of three averages of ``n`` calls, in ms."""
    fn()
    best = float("inf")
    for _ in range(3):
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        for _ in range(n):
            fn()
        torch.cuda.synchronize()
        best = min(best, (time.perf_counter() - t0) * 1e3 / n)
    return best


def prefill_ms(engine, prompts: List[torch.Tensor], n: int) -> float:
    def once():
        engine.reset()
        if engine.B == 1:
            engine.prefill(prompts[0])
        else:
            engine.prefill_batch(prompts)
    return _time(once, n)


def decode_ms(engine, prompts, n: int) -> float:
    engine.eos = -1
    engine.reset()
    if engine.B == 1:
        engine.prefill(prompts[0])
    else:
        engine.prefill_batch(prompts)
    return _time(lambda: engine.decode_step(True), n)


def run(sizes=("1b", "7b"), pairs: int = 4, prompts=(512, 4096), packs=((8, 512),), streams=(1, 8, 32), context: int = 1024,
        steps: int = 40, only: str = "both", design: str = "nusitar", emit=print) -> List[dict]:
    from ..models import LayeredConfig, LayeredDecoder
    from ..parallel.tp import TensorParallelEngine
    from ..runtime.layered_engine import LayeredEngine
    dev = torch.device("cuda:0")
    vocab = 32000
    out: List[dict] = []
    for size in sizes:
        cfg = CONFIGS[design](size, pairs, vocab)
        model = LayeredDecoder.from_config(LayeredConfig(cfg), torch.bfloat16, dev, seed=0)
        llama = llama_like(size, int(layer_params(model)), vocab, dev)
        width = cfg["width"]
        models = {design: model, "llama": llama}
        params = {k: int(layer_params(m)) + vocab * width for k, m in models.items()}
        which = [k for k in models if only in ("both", k)]

        def ids(n):
            return torch.randint(0, vocab, (n,), device=dev, dtype=torch.int32)

        def emb(n):
            return (torch.randn(n, width, device=dev) * 0.02).to(torch.bfloat16)

        def engine(k, batch, length):
            kw = dict(max_len=length + 256, max_batch=batch, max_new_tokens=512)
            if k == design:
                return LayeredEngine(model, **kw)
            return llama.engine(max_len=length + 256, max_new_tokens=512) if batch == 1 else TensorParallelEngine(llama, None, **kw)

        def row(kind, batch, length, fn):
            r = {"size": size, "pass": kind, "batch": batch, "tokens": length}
            for k in which:
                llama._engine = None
                e = engine(k, batch, length)
                ms = fn(e, [(ids if k == design else emb)(length) for _ in range(batch)])
                work = params[k] * 2
                if kind == "prefill":
                    r[k] = {"ms": round(ms, 3), "tok_s": round(batch * length / ms * 1e3),
                            "tflops": round((params[k] - vocab * width) * 2 * batch * length / ms / 1e9, 1)}
                else:
                    r[k] = {"ms": round(ms, 4), "tok_s": round(batch / ms * 1e3), "weight_tb_s": round(work / ms / 1e9, 2)}
                del e
                torch.cuda.empty_cache()
            out.append(r)
            emit(json.dumps(r))
        for n in prompts:
            row("prefill", 1, n, lambda e, p: prefill_ms(e, p, 8))
        for b, n in packs:
            row("prefill", b, n, lambda e, p: prefill_ms(e, p, 8))
        for b in streams:
            row("decode", b, context, lambda e, p: decode_ms(e, p, steps))
        emit(json.dumps({"size": size, "layers": {design: 2 * pairs, "llama": llama.config.num_hidden_layers},
                         "params": {k: v for k, v in params.items()}}))
        del model, llama, models
        torch.cuda.empty_cache()
    return out
