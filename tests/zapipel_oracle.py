"""Plain, slow oracle of the Zapipel decoder: one function per mechanism.  Works in whatever dtype its
inputs have (tests use float64) and shares no code with the package: it reads the configuration dictionary
and a name -> tensor mapping."""
import torch


def rms(x, eps, w):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def layer_norm(x, eps, w):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w


def silu(z):
    return z * torch.sigmoid(z)


def softcap(z, scale, cap):
    return cap * torch.tanh(z * scale / cap)


def causal_attention(q, k, v, scale):
    """``q, k [T, H, D]``, ``v [T, H, V]``: position i sees 0 .. i, softmax."""
    out = []
    for i in range(q.shape[0]):
        s = (k[:i + 1] * q[i]).sum(-1) * scale          # [i + 1, H]
        w = torch.exp(s - s.max(0).values)
        w = w / w.sum(0)
        out.append((w[:, :, None] * v[:i + 1]).sum(0))
    return torch.stack(out)


def latent(h, P, eps):
    """What a layer caches per token."""
    return rms(h @ P("dkv").T, eps, P("dkv.norm"))


def latent_attention(h, c, P, cfg, eps):
    """``c``: the latents of the layer that owns them."""
    T, H, D, V = h.shape[0], cfg["heads"], cfg["dim"], cfg["vdim"]
    q = (rms(h @ P("dq").T, eps, P("dq.norm")) @ P("uq").T).reshape(T, H, D)
    k = (c @ P("uk").T).reshape(T, H, D)
    v = (c @ P("uv").T).reshape(T, H, V)
    o = causal_attention(q, k, v, cfg["scale"])
    o = o * torch.sigmoid(h @ P("g").T)[:, :, None]
    return o.reshape(T, H * V) @ P("o").T


def gated_unit(h, P, pre=""):
    return (silu(h @ P(pre + "gate").T) * (h @ P(pre + "up").T)) @ P(pre + "down").T


def route(z, top):
    """Chosen experts and their weights for router logits ``z [T, E]``."""
    best, which = torch.sort(z, dim=-1, descending=True, stable=True)
    best, which = best[:, :top], which[:, :top]
    w = torch.exp(best - best[:, :1])
    return which, w / w.sum(-1, keepdim=True)


def mixture(h, P, top):
    which, w = route(h @ P("router").T + P("router.b"), top)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, we in zip(which[t].tolist(), w[t]):
            out[t] = out[t] + we * gated_unit(h[t], P, "e%d." % e)
    return out


def forward(cfg, weights, tokens, keep_layers=False):
    """Logits ``[T, vocab]`` of one sequence (and the residual stream after every layer)."""
    eps = cfg["norm"]["eps"]
    x = weights["embed"][torch.as_tensor(tokens).long()]
    stream, latents = [], {}
    for n, layer in enumerate(cfg["layers"]):
        def P(name, pre="l%d." % n):
            return weights[pre + name]
        mix, mlp = layer["mixer"], layer["mlp"]
        h = layer_norm(x, eps, P("norm1"))
        if mix.get("kv_from") is None:
            latents[n] = latent(h, lambda s: P("mix." + s), eps)
        c = latents[n if mix.get("kv_from") is None else mix["kv_from"]]
        x = x + layer_norm(latent_attention(h, c, lambda s: P("mix." + s), mix, eps), eps, P("norm1b"))
        if mlp is not None:
            h = layer_norm(x, eps, P("norm2"))
            if mlp["kind"] == "moe":
                y = mixture(h, lambda s: P("mlp." + s), mlp["router"]["top"])
            else:
                y = gated_unit(h, lambda s: P("mlp." + s))
            x = x + layer_norm(y, eps, P("norm2b"))
        stream.append(x)
    logits = softcap(layer_norm(x, eps, weights["final.norm"]) @ weights["head"].T, cfg["logit_scale"], cfg["logit_softcap"])
    return (logits, torch.stack(stream)) if keep_layers else logits
