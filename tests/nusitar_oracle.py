"""Plain, slow oracle of the Nusitar decoder: one function per mechanism, token by token where a
mechanism is a recurrence.  Works in whatever dtype its inputs have (tests use float64) and shares
no code with the package: it reads the configuration dictionary and a name -> tensor mapping."""
import math

import torch


def rms(x, eps, w=None, parts=1):
    """RMS norm of the last dimension in ``parts`` equal parts, times ``w``."""
    shape = x.shape
    x = x.reshape(*shape[:-1], parts, shape[-1] // parts)
    x = x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)
    x = x.reshape(shape)
    return x if w is None else x * w


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def rotate(x, positions, dims, base):
    """Rotate-half rotary embedding of the first ``dims`` of every head of ``x [T, H, D]``."""
    half = dims // 2
    freq = base ** (-2.0 * torch.arange(half, dtype=torch.float64) / dims)
    ang = positions.to(torch.float64)[:, None] * freq[None]
    c, s = ang.cos().to(x.dtype)[:, None], ang.sin().to(x.dtype)[:, None]
    u, v, rest = x[..., :half], x[..., half:dims], x[..., dims:]
    return torch.cat([u * c - v * s, v * c + u * s, rest], -1)


def chunked_attention(q, k, v, scale, size):
    """Causal softmax attention inside blocks of ``size`` positions.  ``q [T, H, D]``, ``k [T, G, D]``."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = q.new_zeros(T, H, v.shape[-1])
    for i in range(T):
        lo = i // size * size
        for h in range(H):
            g = h // (H // G)
            w = torch.softmax((k[lo:i + 1, g] @ q[i, h]) * scale, 0)
            out[i, h] = w @ v[lo:i + 1, g]
    return out


def attention_branch(h, P, cfg, eps):
    T = h.shape[0]
    H, G, D, V = cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    q = rms(h @ P("q").T, eps, P("q.norm")).reshape(T, H, D)
    k = rms(h @ P("k").T, eps, P("k.norm")).reshape(T, G, D)
    v = (h @ P("v").T).reshape(T, G, V)
    pos = torch.arange(T)
    q = rotate(q, pos, cfg["rot"]["dims"], cfg["rot"]["base"])
    k = rotate(k, pos, cfg["rot"]["dims"], cfg["rot"]["base"])
    o = chunked_attention(q, k, v, cfg["scale"], cfg["mask"]["size"])
    return o.reshape(T, H * V) @ P("o").T


def mlstm_scan(q, k, v, i, f):
    """Matrix memory with a running maximum.  ``q, k [T, H, N]``, ``v [T, H, V]``, log gates ``[T, H]``."""
    T, H, N = q.shape
    S = q.new_zeros(H, N, v.shape[-1])
    n = q.new_zeros(H, N)
    m = q.new_zeros(H)
    out = []
    for t in range(T):
        new = torch.maximum(f[t] + m, i[t])
        keep, add = torch.exp(f[t] + m - new), torch.exp(i[t] - new)
        m = new
        S = keep[:, None, None] * S + add[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = keep[:, None] * n + add[:, None] * k[t]
        top = (S * q[t][:, :, None]).sum(1)
        bottom = torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        out.append(top / bottom[:, None])
    return torch.stack(out)


def mlstm_branch(h, P, cfg, eps):
    T = h.shape[0]
    H, N, V, cap = cfg["heads"], cfg["dim"], cfg["vdim"], cfg["gate_cap"]
    q = (h @ P("q").T).reshape(T, H, N) * N ** -0.5
    k = (h @ P("k").T).reshape(T, H, N)
    v = (h @ P("v").T).reshape(T, H, V)
    i = cap * torch.tanh((h @ P("i").T + P("i.b")) / cap)
    f = -softplus(-cap * torch.tanh((h @ P("f").T + P("f.b")) / cap))
    o = rms(mlstm_scan(q, k, v, i, f), eps).reshape(T, H * V)
    return (o * P("norm") * torch.sigmoid(h @ P("g").T)) @ P("o").T


def parallel_mixer(h, P, cfg, eps):
    a = attention_branch(h, lambda n: P("left." + n), cfg["left"], eps)
    b = mlstm_branch(h, lambda n: P("right." + n), cfg["right"], eps)
    return 0.5 * (rms(a, eps, P("left.out")) + rms(b, eps, P("right.out")))


def causal_conv(x, w, b):
    """Per-channel convolution over the current and earlier tokens of ``x [T, C]``; ``w [C, taps]``."""
    taps = w.shape[1]
    y = b.expand(x.shape).clone()
    for t in range(x.shape[0]):
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                y[t] = y[t] + w[:, j] * x[s]
    return y


def ssd_scan(x, B, C, dt, A_log, D):
    """Mamba-2 recurrence.  ``x [T, H, V]``, ``B, C [T, G, N]``, ``dt [T, H]``."""
    T, H, V = x.shape
    G, N = B.shape[1:]
    per = H // G
    S = x.new_zeros(H, N, V)
    out = []
    for t in range(T):
        b, c = B[t].repeat_interleave(per, 0), C[t].repeat_interleave(per, 0)
        S = torch.exp(-torch.exp(A_log) * dt[t])[:, None, None] * S \
            + dt[t][:, None, None] * b[:, :, None] * x[t][:, None, :]
        out.append((S * c[:, :, None]).sum(1) + D[:, None] * x[t])
    return torch.stack(out)


def mamba2_mixer(h, P, cfg, eps):
    T = h.shape[0]
    H, V, N, G = cfg["heads"], cfg["vdim"], cfg["state"], cfg["groups"]
    inner = H * V
    z, xbc, dt = (h @ P("in").T).split([inner, inner + 2 * G * N, H], -1)
    xbc = silu(causal_conv(xbc, P("conv"), P("conv.b")))
    x, B, C = xbc.split([inner, G * N, G * N], -1)
    y = ssd_scan(x.reshape(T, H, V), B.reshape(T, G, N), C.reshape(T, G, N), softplus(dt + P("dt_bias")),
                 P("A_log"), P("D"))
    y = rms(y.reshape(T, inner) * silu(z), eps, P("norm"), cfg["norm_groups"])
    return y @ P("o").T


MIXERS = {"mamba2": mamba2_mixer, "parallel": parallel_mixer}


def forward(cfg, weights, tokens, keep_layers=False):
    """Logits ``[T, vocab]`` of one sequence (and the residual stream after every layer)."""
    eps = cfg["norm"]["eps"]
    x = weights["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
    stream = []
    for n, layer in enumerate(cfg["layers"]):
        def P(name, pre="l%d." % n):
            return weights[pre + name]
        x = x + MIXERS[layer["type"]](rms(x, eps, P("norm1")), lambda s: P("mix." + s), layer["mixer"], eps)
        if layer["mlp"] is not None:
            h = rms(x, eps, P("norm2"))
            x = x + (gelu_tanh(h @ P("mlp.gate").T) * (h @ P("mlp.up").T)) @ P("mlp.down").T
        stream.append(x)
    logits = rms(x, eps, weights["final.norm"]) @ weights["head"].T
    return (logits, torch.stack(stream)) if keep_layers else logits
