"""Small Nusitar configurations and models for the tests."""
import torch

import nusitar_oracle as oracle
from eventgpt_amd.models import LayeredConfig, LayeredDecoder


def attention(heads=6, kv_heads=2, dim=20, vdim=28, scale=0.31, dims=12, base=700.0, size=13):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
            "rot": {"dims": dims, "base": base}, "mask": {"size": size}}


def memory(heads=3, dim=40, vdim=24, gate_cap=4.0):
    return {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": gate_cap}


def parallel(left=None, right=None, ff=72):
    return {"type": "parallel", "mixer": {"left": left or attention(), "right": right or memory()},
            "mlp": ff and {"kind": "dense", "ff": ff}}


def mamba(heads=6, groups=3, state=24, vdim=20, conv=3, norm_groups=5, ff=None):
    return {"type": "mamba2", "mixer": {"heads": heads, "groups": groups, "state": state, "vdim": vdim, "conv": conv,
                                        "norm_groups": norm_groups}, "mlp": ff and {"kind": "dense", "ff": ff}}


def config(layers, vocab=83, width=100, eps=3e-5, scale=1.7):
    return {"architecture": "Nusitar", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"scale": scale}, "layers": layers}


# every mechanism with sizes that are not multiples of anything, unequal q / v head sizes, layers that differ
MIXED = config([
    mamba(),
    parallel(),
    parallel(attention(heads=5, kv_heads=5, dim=33, vdim=16, dims=0, size=7, scale=0.12), memory(heads=2, dim=16, vdim=70, gate_cap=9.0), None),
    mamba(heads=4, groups=1, state=40, vdim=36, conv=5, norm_groups=1, ff=52),
    parallel(attention(heads=4, kv_heads=1, dim=72, vdim=80, dims=72, size=29, scale=0.09), memory(heads=1, dim=9, vdim=33), 33),
    mamba(heads=2, groups=2, state=8, vdim=5, conv=2, norm_groups=2),
])


def build(cfg=MIXED, dtype=torch.float32, device="cpu", seed=1):
    """A model with random weights that bf16 holds exactly.  The 32-bit one has wide open input gates as well: its
    matrix memories divide by |n . q| near zero at some tokens, which 16-bit activations would blow up."""
    m = LayeredDecoder.from_config(LayeredConfig(cfg), torch.bfloat16, "cpu", seed)
    if dtype == torch.float32:
        for n, t in m.tensors.items():
            if n.endswith(".i.b"):
                t += 3
    out = LayeredDecoder(m.config, dtype, device)
    for n, t in m.tensors.items():
        out.tensors[n].copy_(t)
    return out


def weights(model):
    return {n: t.detach().cpu().double() for n, t in model.tensors.items()}


def oracle_logits(model, tokens):
    return oracle.forward(model.config.raw, weights(model), tokens)


def prompt(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed), dtype=torch.int32)


def rel_err(got, want):
    """Root mean square of the difference over that of the reference, the worst row."""
    got, want = got.double().cpu(), want.double().cpu()
    d = (got - want).pow(2).mean(-1).sqrt()
    return float((d / want.pow(2).mean().sqrt()).max())
