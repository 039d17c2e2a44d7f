"""Small Zapipel configurations and models for the tests."""
import copy

import torch

import zapipel_oracle as oracle
from _nusitar import prompt, rel_err  # noqa: F401  (shared helpers)
from eventgpt_amd.models import LayeredConfig, LayeredDecoder


def layer(heads=5, dim=20, vdim=28, kv_rank=40, q_rank=24, scale=0.31, kv_from=None, mlp=None):
    mix = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank, "scale": scale}
    if kv_from is not None:
        mix["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": mix, "mlp": mlp}


def dense(ff=52):
    return {"kind": "dense", "ff": ff}


def moe(experts=5, top=3, ff=24):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def config(layers, vocab=83, width=100, eps=3e-4, scale=0.7, cap=4.0):
    return {"architecture": "Zapipel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_scale": scale,
            "logit_softcap": cap, "layers": layers}


# sizes that are multiples of nothing, unequal query / value sizes, latents that later layers read with other heads and
# sizes, a layer without a feed-forward, one expert, every expert, more heads than a tile
MIXED = config([
    layer(mlp=moe()),
    layer(heads=18, dim=33, vdim=16, kv_rank=100, q_rank=70, scale=0.12, mlp=dense(72)),
    layer(heads=3, dim=72, vdim=80, q_rank=9, scale=0.05, kv_from=0),
    layer(heads=1, dim=8, vdim=5, kv_rank=100, q_rank=130, scale=0.9, kv_from=1, mlp=moe(1, 1, 33)),
    layer(heads=7, dim=65, vdim=64, kv_rank=7, q_rank=33, scale=0.2, mlp=moe(9, 1, 8)),
    layer(heads=4, kv_from=0, scale=1.0, mlp=moe(6, 6, 40)),
])
SMALL = config([layer(heads=2, mlp=dense(40)), layer(heads=3, kv_from=0, mlp=moe(4, 2, 16)), layer(kv_rank=70)], vocab=50, width=72,
               scale=1.3, cap=9.0)
WIDE = config([layer(heads=20, dim=128, vdim=128, kv_rank=300, q_rank=200, scale=0.09, mlp=dense(320)),
               layer(heads=16, dim=100, vdim=128, kv_rank=300, q_rank=64, kv_from=0, scale=0.1, mlp=moe(4, 4, 96))], vocab=120, width=264)


def all_chosen(cfg):
    """The same with every expert chosen: no choice that rounding could turn."""
    cfg = copy.deepcopy(cfg)
    for e in cfg["layers"]:
        if e["mlp"] is not None and e["mlp"]["kind"] == "moe":
            e["mlp"]["router"]["top"] = e["mlp"]["router"]["experts"]
    return cfg


def build(cfg=MIXED, dtype=torch.float32, device="cpu", seed=1):
    """A model with random weights that bf16 holds exactly."""
    m = LayeredDecoder.from_config(LayeredConfig(cfg), torch.bfloat16, "cpu", seed)
    out = LayeredDecoder(m.config, dtype, device)
    for n, t in m.tensors.items():
        out.tensors[n].copy_(t)
    return out


def weights(model):
    return {n: t.detach().cpu().double() for n, t in model.tensors.items()}


def oracle_logits(model, tokens):
    return oracle.forward(model.config.raw, weights(model), tokens)


def row_err(got, want):
    """The worst row's root mean square of the difference over the row's own."""
    got, want = got.double().cpu(), want.double().cpu()
    return float(((got - want).pow(2).mean(-1) / want.pow(2).mean(-1)).max()) ** 0.5
