"""Layered decoder kernels and engine on the GPU against the plain oracle (tests/nusitar_oracle.py)."""
import copy

import pytest
import torch

import _nusitar as N
import nusitar_oracle as oracle
from eventgpt_amd.models import LayeredConfig, LayeredDecoder
from eventgpt_amd.runtime.mixers import RowBatch, Sequence_

pytestmark = pytest.mark.gpu

DTYPES = [torch.float32, torch.bfloat16]
TOL = {torch.float32: 2e-5, torch.bfloat16: 2e-2}       # one mechanism, relative to the output's rms
MODEL_TOL = {torch.float32: 1e-4, torch.bfloat16: 8e-2}  # logits of a whole model


@pytest.fixture(scope="module")
def raw(dev):
    from eventgpt_amd.ops import layered
    return layered.raw


def rnd(*shape, seed=0, scale=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64) * scale


def typed(t, dtype, dev):
    """``(device tensor, the same values in double)``."""
    d = t.to(dtype)
    return d.to(dev).contiguous(), d.double()


# ------------------------------------------------------------------ one mechanism at a time
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("m,n,k", [(1, 8, 64), (5, 136, 192), (70, 72, 64), (130, 200, 320), (33, 1000, 128)])
def test_projection(raw, dev, dtype, m, n, k):
    x, xr = typed(rnd(m, k), dtype, dev)
    w, wr = typed(rnd(n, k, seed=1, scale=k ** -0.5), dtype, dev)
    want = xr @ wr.T
    tol = 2e-6 if dtype == torch.float32 else 1e-5
    assert N.rel_err(raw.linear(x, w, True), want) < tol
    assert N.rel_err(raw.linear_slabs(x, w).sum(0), want) < tol
    if dtype == torch.bfloat16:
        assert N.rel_err(raw.linear(x, w, False), want) < 4e-3


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [100, 64, 9000])
def test_residual_rows(raw, dev, dtype, width):
    rows, ld, eps, f32 = 5, -(-width // 64) * 64, 3e-3, dtype == torch.float32

    def padded(t):
        out = torch.zeros(*t.shape[:-1], ld, dtype=t.dtype)
        out[..., :width] = t
        return out
    x, a, b, c = (rnd(rows, width, seed=s).float() for s in range(4))
    w, wa, wb = (1 + 0.3 * rnd(width, seed=10 + s).float() for s in range(3))
    X, A, B, C, W, WA, WB = (padded(t).to(dev) for t in (x, a, b, c, w, wa, wb))
    x, a, b, c, w, wa, wb = (t.double() for t in (x, a, b, c, w, wa, wb))
    tol = 1e-6 if f32 else 4e-3
    sel = torch.tensor([4, 0, 4], dtype=torch.int32, device=dev)
    assert N.rel_err(raw.norm_rows(X, sel, W, width, eps, f32)[:, :width], oracle.rms(x, eps, w)[[4, 0, 4]]) < tol
    # slabs are summed, the stream stays fp32
    Y = X.clone()
    xn = raw.add_norm_rows_(Y, torch.stack([A, C]), W, width, eps, f32)
    assert N.rel_err(Y[:, :width], x + a + c) < 1e-6 and N.rel_err(xn[:, :width], oracle.rms(x + a + c, eps, w)) < tol
    assert xn.dtype == dtype and float(xn[:, width:].float().abs().sum()) == 0
    Y = X.clone()
    xn = raw.merge_norm_rows_(Y, A, torch.stack([B, C]), WA, WB, W, width, eps, f32)
    want = x + 0.5 * (oracle.rms(a, eps, wa) + oracle.rms(b + c, eps, wb))
    assert N.rel_err(Y[:, :width], want) < 1e-6 and N.rel_err(xn[:, :width], oracle.rms(want, eps, w)) < tol
    Y = X.clone()
    assert raw.merge_norm_rows_(Y, A, B, WA, WB, None, width, eps, f32).numel() == 0


@pytest.mark.parametrize("dtype", DTYPES)
def test_embedding_and_commit(raw, dev, dtype):
    e, er = typed(rnd(11, 64), dtype, dev)
    tok = torch.tensor([3, 10, 0], dtype=torch.int32, device=dev)
    assert N.rel_err(raw.embed_rows(tok, e, 2.5), er[[3, 10, 0]] * 2.5) < 1e-6
    i = dict(dtype=torch.int32, device=dev)
    x, out = torch.zeros(3, 64, device=dev), torch.zeros(3, 4, **i)
    step, pos, done, cur = torch.tensor([0, 2, 1], **i), torch.tensor([5, 6, 7], **i), torch.zeros(3, **i), torch.zeros(3, **i)
    raw.commit_rows_(None, tok, e, 2.5, x, out, step, pos, done, cur, 10, torch.tensor([1, 1, 0], **i))
    assert out.tolist() == [[3, 0, 0, 0], [0, 0, 10, 0], [0, 0, 0, 0]]
    assert step.tolist() == [1, 3, 1] and pos.tolist() == [6, 7, 7] and done.tolist() == [0, 1, 0] and cur.tolist() == [3, 10, 0]
    assert N.rel_err(x[:2], er[[3, 10]] * 2.5) < 1e-6 and float(x[2].abs().sum()) == 0


def test_greedy_commit_takes_the_first_maximum(raw, dev):
    V = 9001
    lg = torch.full((4, V + 7), -5.0)
    lg[0, 8999] = 9
    lg[1, 40] = lg[1, 3] = lg[1, 4099] = 2
    lg[2, V + 2] = 9                                 # outside the vocabulary
    lg[2, 70] = 1
    lg[3, 5] = float("nan")
    lg[3, 9000] = 0
    i = dict(dtype=torch.int32, device=dev)
    tok, out, st = torch.zeros(4, **i), torch.zeros(4, 2, **i), [torch.zeros(4, **i) for _ in range(4)]
    e = torch.arange(V, dtype=torch.float32)[:, None].repeat(1, 64).to(dev)
    x = torch.zeros(4, 64, device=dev)
    raw.commit_rows_(lg.to(dev)[:, :V], tok, e, 0.5, x, out, *st, -1, None)
    assert tok.tolist() == [8999, 3, 70, 9000] and out[:, 0].tolist() == tok.tolist()
    assert x[:, 63].tolist() == [t / 2 for t in tok.tolist()] and st[1].tolist() == [1] * 4


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,v,vp,parts,before", [(3, 24, 32, 3, False), (6, 20, 32, 5, True), (4, 48, 64, 1, True),
                                                     (5, 70, 128, 7, True), (2, 64, 64, 2, False)])
def test_group_norm_with_gate(raw, dev, dtype, heads, v, vp, parts, before):
    rows, slots, eps = 4, heads * vp, 1e-3
    y, gate, w = torch.zeros(rows, heads, vp), torch.zeros(rows, 8 + slots), torch.zeros(heads, vp)
    y[..., :v] = rnd(rows, heads, v).float()
    gate[:, 8:] = rnd(rows, slots, seed=1).float()
    w[:, :v] = 1 + 0.2 * rnd(heads, v, seed=2).float()
    (yd, yr), (gd, gr) = typed(y, dtype, dev), typed(gate, dtype, dev)
    o = raw.group_norm_rows(yd.view(rows, -1), gd, 8, 1 if before else 2, w.to(dev), heads, v, vp, parts, slots + 64, eps,
                            dtype == torch.float32)
    real = yr[..., :v].reshape(rows, -1)
    g = gr[:, 8:].view(rows, heads, vp)[..., :v].reshape(rows, -1)
    wr = w[:, :v].reshape(-1).double()
    want = oracle.rms(real * oracle.silu(g), eps, wr, parts) if before else oracle.rms(real, eps, wr, parts) * torch.sigmoid(g)
    got = o[:, :slots].view(rows, heads, vp)
    assert N.rel_err(got[..., :v].reshape(rows, -1), want) < (2e-6 if dtype == torch.float32 else 6e-3)
    assert float(got[..., v:].float().abs().sum()) == 0 and float(o[:, slots:].float().abs().sum()) == 0
    plain = raw.group_norm_rows(y.view(rows, -1).to(dev), None, 0, 0, w.to(dev), heads, v, vp, parts, slots, eps, True)
    assert N.rel_err(plain.view(rows, heads, vp)[..., :v].reshape(rows, -1),
                     oracle.rms(y[..., :v].reshape(rows, -1).double(), eps, wr, parts)) < 2e-6


@pytest.mark.parametrize("dtype", DTYPES)
def test_glu(raw, dev, dtype):
    src, sr = typed(rnd(7, 2 * 72, scale=2), dtype, dev)
    a, b = sr.chunk(2, -1)
    tol = 1e-6 if dtype == torch.float32 else 6e-3
    assert N.rel_err(raw.glu_rows(src, 0, dtype == torch.float32), oracle.gelu_tanh(a) * b) < tol
    assert N.rel_err(raw.glu_rows(src, 1, dtype == torch.float32), oracle.silu(a) * b) < tol
    # projection and gate together: slabs + gate for few rows, the GEMM's epilogue for many
    for m in (3, 40, 300):
        x, xr = typed(rnd(m, 128, seed=3), dtype, dev)
        w, wr = typed(rnd(2 * 192, 128, seed=4, scale=128 ** -0.5), dtype, dev)
        g, u = (xr @ wr.T).chunk(2, -1)
        for act, f in ((0, oracle.gelu_tanh), (1, oracle.silu)):
            assert N.rel_err(raw.linear_glu(x, w, act), f(g) * u) < (3e-6 if dtype == torch.float32 else 8e-3)


@pytest.mark.parametrize("dtype", DTYPES)
def test_recurrence_gates(raw, dev, dtype):
    """Log gates over their whole range: gates at the cap, a forget gate near 0 and near 1, large and tiny dt."""
    x = torch.cat([torch.linspace(-60, 60, 31), torch.linspace(-3, 3, 17)])[:, None].repeat(1, 16).double()
    xd, xr = typed(x, dtype, dev)
    ib, fb = rnd(8).float(), rnd(8, seed=1).float()
    li, lf = raw.mlstm_gates(xd, 0, 8, ib.to(dev), fb.to(dev), 7.0)
    assert torch.allclose(li.cpu().double(), 7 * torch.tanh((xr[:, :8] + ib.double()) / 7), rtol=2e-6, atol=2e-6)
    want = -oracle.softplus(-7 * torch.tanh((xr[:, 8:] + fb.double()) / 7))
    assert torch.allclose(lf.cpu().double(), want, rtol=4e-6, atol=1e-8)
    ld, dt = raw.ssd_gates(xd, 8, fb.to(dev), ib.to(dev))
    want = oracle.softplus(xr[:, 8:] + fb.double())
    assert torch.allclose(dt.cpu().double(), want, rtol=4e-6, atol=0)
    assert torch.allclose(ld.cpu().double(), -torch.exp(ib.double()) * want, rtol=4e-6, atol=0)


def pack(lens, starts=None):
    seqs, row = [], 0
    for i, n in enumerate(lens):
        seqs.append(Sequence_(i, row, n, 0 if starts is None else starts[i]))
        row += n
    return seqs


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("taps", [1, 2, 4, 7])
def test_convolution(raw, dev, dtype, taps):
    """Whole sequences, portions (also shorter than the taps) and single tokens give the same rows."""
    C, lens = 72, [1, 9, 30]
    w, b = rnd(C, taps, seed=1).float(), rnd(C, seed=2).float()
    x = [typed(rnd(n, C, seed=5 + n), dtype, dev) for n in lens]
    want = [oracle.silu(oracle.causal_conv(r, w.double(), b.double())) for _, r in x]
    wd, bd = w.to(dev), b.to(dev)

    def run(cuts):
        ring = torch.full((len(lens), taps, C), 77.0, dtype=dtype, device=dev)     # stale state of earlier owners
        got, at = [[] for _ in lens], [0] * len(lens)
        for cut in cuts:
            live = [i for i in range(len(lens)) if at[i] < lens[i]]
            n = {i: min(cut, lens[i] - at[i]) for i in live}
            src = torch.cat([x[i][0][at[i]:at[i] + n[i]] for i in live])
            seqs, row = [], 0
            for i in live:
                seqs.append(Sequence_(i, row, n[i], at[i]))
                row += n[i]
            rb = RowBatch(dev, False, seqs=seqs)
            o = raw.conv_rows_(src, 0, wd, bd, ring, rb.slot, rb.pos, rb.first)
            raw.conv_tail_(src, 0, ring, rb.tails)
            for s in seqs:
                got[s.slot].append(o[s.row0:s.row0 + s.rows])
                at[s.slot] += s.rows
        return [torch.cat(g) for g in got]
    tol = 2e-6 if dtype == torch.float32 else 6e-3
    for cuts in ([100], [2] * 15, [5] * 6, [1] * 30, [3, 1, 100]):
        for g, r in zip(run(cuts), want):
            assert N.rel_err(g, r) < tol


def scan_case(kind, dtype, dev, lens, H, per_group, Nn, V, seed=0):
    """Inputs of a recurrence and its oracle outputs per sequence."""
    T, G = sum(lens), H // per_group
    # (the matrix memory divides by |n . q|: an offset keeps it away from zero, where any rounding blows up)
    off = 0.8 if kind == "mlstm" else 0.0
    q, qr = typed((rnd(T, G, Nn, seed=seed) + off) * Nn ** -0.25, dtype, dev)
    k, kr = typed((rnd(T, G, Nn, seed=seed + 1) + off) * Nn ** -0.25, dtype, dev)
    v, vr = typed(rnd(T, H, V, seed=seed + 2), dtype, dev)
    want, at = [], 0
    if kind == "ssd":
        dt = torch.nn.functional.softplus(rnd(T, H, seed=seed + 3)).float()
        a_log, skip = (rnd(H, seed=seed + 4) - 1.5).float(), rnd(H, seed=seed + 5).float()
        ld = (-torch.exp(a_log.double()) * dt.double()).float()
        for n in lens:
            s = slice(at, at + n)
            want.append(oracle.ssd_scan(vr[s], kr[s], qr[s], dt[s].double(), a_log.double(), skip.double()))
            at += n
        gates = (ld.to(dev), None, dt.to(dev), skip.to(dev))
        scale = 1.0
    else:
        li = (3 * rnd(T, H, seed=seed + 3)).float()
        lf = -torch.nn.functional.softplus(-(2 * rnd(T, H, seed=seed + 4) + 2)).float()
        scale = 0.7
        for n in lens:
            s = slice(at, at + n)
            want.append(oracle.mlstm_scan(qr[s] * scale, kr[s], vr[s], li[s].double(), lf[s].double()))
            at += n
        gates = (lf.to(dev), li.to(dev), None, None)
    return q.view(T, -1), k.view(T, -1), v.view(T, -1), gates, scale, want


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind,H,per_group,Nn,V", [("ssd", 4, 2, 32, 64), ("ssd", 3, 3, 96, 32), ("ssd", 2, 1, 128, 64),
                                                   ("mlstm", 2, 1, 32, 32), ("mlstm", 3, 1, 160, 128), ("mlstm", 1, 1, 64, 192)])
def test_recurrence(raw, dev, dtype, kind, H, per_group, Nn, V):
    """Unequal sequences in one pack, in portions (whole chunks, two tokens, single ones, across chunk borders), from
    states that hold an earlier owner's values."""
    lens = [1, 63, 64, 65, 128, 129, 300]
    q, k, v, gates, scale, want = scan_case(kind, dtype, dev, lens, H, per_group, Nn, V)
    offs = [sum(lens[:i]) for i in range(len(lens))]
    B = len(lens)
    tol = TOL[dtype]

    def state():
        f = dict(device=dev, dtype=torch.float32)
        S = torch.full((B, H, V, Nn), 7.0, **f)
        return (S, None, None) if kind == "ssd" else (S, torch.full((2, B, H, Nn), 7.0, **f), torch.full((2, B, H), 7.0, **f))

    def rows(t, idx):
        return None if t is None else (t if t.dim() == 1 else t[idx].contiguous())
    for cuts in ([1000], [64] * 5, [128] * 3, [2] * 150, [1] * 300, [37] * 9, [130, 3, 170]):
        st, at, got = state(), [0] * B, [[] for _ in lens]
        for cut in cuts:
            seqs, idx, row = [], [], 0
            for i in range(B):
                n = min(cut, lens[i] - at[i])
                if n > 0:
                    seqs.append(Sequence_(i, row, n, at[i]))
                    idx += range(offs[i] + at[i], offs[i] + at[i] + n)
                    row += n
            if not seqs:
                break
            rb = RowBatch(dev, False, seqs=seqs, scan_chunk=raw.scan_chunk(dtype == torch.float32))
            ix = torch.tensor(idx, device=dev)
            o = raw.scan_prefill_(q[ix], k[ix], v[ix], H, per_group, Nn, V, scale, *(rows(g, ix) for g in gates), *st,
                                  rb.chunks, rb.scan_seqs)
            for s in seqs:
                got[s.slot].append(o[s.row0:s.row0 + s.rows])
                at[s.slot] += s.rows
        for g, w in zip(got, want):
            assert N.rel_err(torch.cat(g), w.reshape(w.shape[0], -1)) < tol, cuts


def step_rows(dtype, dev, cols):
    """Projection rows of a decode step: values that T holds, as one fp32 matrix and as three slabs that sum to it."""
    x = torch.cat(cols, -1)
    pad = torch.zeros(x.shape[0], -x.shape[1] % 8)
    x = torch.cat([x, pad], -1).to(dev)
    a = torch.round(x * 0.5 * 256) / 256
    return x, torch.stack([a, x - a, torch.zeros_like(x)])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,Nn,V,v_used", [(4, 2, 32, 64, 64), (3, 1, 96, 32, 20), (2, 2, 128, 128, 128)])
def test_ssd_decode_step(raw, dev, dtype, H, G, Nn, V, v_used):
    """Convolution, gates, recurrence and output gate of single tokens; unequal sequences, a slot that is parked now and
    then, stale state of an earlier owner, rows as a matrix and as slabs."""
    taps, lens, T = 3, [9, 5], 9
    inner, C = H * V, H * V + 2 * G * Nn
    f = dict(dtype=torch.float32, device=dev)
    z, xbc = typed(rnd(2, T, inner), dtype, "cpu")[0].float(), typed(rnd(2, T, C, seed=1), dtype, "cpu")[0].float()
    dt = rnd(2, T, H, seed=2).float()
    cw, cb = rnd(C, taps, seed=3).float(), rnd(C, seed=4).float()
    bias, a_log, skip = (rnd(H, seed=5 + i).float() for i in range(3))
    S, ring = torch.full((2, H, V, Nn), 9.0, **f), torch.full((2, taps, C), 9.0, dtype=dtype, device=dev)
    want = []
    for b in range(2):
        c = oracle.silu(oracle.causal_conv(xbc[b].double(), cw.double(), cb.double()))
        c = c.to(dtype).double()
        x, bb, cc = c.split([inner, G * Nn, G * Nn], -1)
        y = oracle.ssd_scan(x.reshape(T, H, V), bb.reshape(T, G, Nn), cc.reshape(T, G, Nn),
                            oracle.softplus(dt[b].double() + bias.double()), a_log.double(), skip.double())
        want.append(y.reshape(T, inner) * oracle.silu(z[b].double()))
    dims = [0, inner, inner + C, H, G, Nn, V]
    args = [t.to(dev) for t in (cw, cb)] + [ring] + [t.to(dev) for t in (bias, a_log, skip)]
    for t in range(T):
        live = torch.tensor([1, int(t < lens[1])], dtype=torch.int32, device=dev)
        pos = torch.full((2,), t, dtype=torch.int32, device=dev)
        rows = step_rows(dtype, dev, [z[:, t], xbc[:, t], dt[:, t]])
        off = torch.zeros(2, dtype=torch.int32, device=dev)
        before = S.clone(), ring.clone()
        raw.ssd_step_(rows[0] + 1, dims, *args, S, pos, off)
        assert torch.equal(before[0], S) and torch.equal(before[1], ring)
        o = raw.ssd_step_(rows[t % 2], dims, *args, S, pos, live)
        for b in range(2):
            if t < lens[b]:
                assert N.rel_err(o[b:b + 1], want[b][t:t + 1]) < (1e-5 if dtype == torch.float32 else 1e-2), (t, b)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("Hr,Nn,V", [(3, 32, 64), (1, 160, 32), (2, 64, 192)])
def test_parallel_decode_step(raw, dev, dtype, Hr, Nn, V):
    """Attention heads (norm, rotation, cache append) and matrix memory of single tokens from one set of rows."""
    H, G, d, D, dims, cap, eps, T, lens, mcap = 6, 2, 20, 64, 12, 4, 1e-3, 11, [11, 6], 5.0
    f = dict(dtype=torch.float32, device=dev)
    att = torch.zeros(2, T, H + 2 * G, D)
    att[..., :d] = rnd(2, T, H + 2 * G, d).float()
    att = att.to(dtype).float()
    q, k = (typed(rnd(2, T, Hr, Nn, seed=s, scale=Nn ** -0.25), dtype, "cpu")[0].float() for s in (1, 2))
    v = typed(rnd(2, T, Hr, V, seed=3), dtype, "cpu")[0].float()
    gi, gf = 3 * rnd(2, T, Hr, seed=4).float(), 2 + rnd(2, T, Hr, seed=5).float()
    ib, fb = rnd(Hr, seed=6).float(), rnd(Hr, seed=7).float()
    qw, kw = torch.zeros(H, D), torch.zeros(G, D)
    qw[:, :d], kw[:, :d] = 1 + 0.2 * rnd(H, d, seed=8).float(), 1 + 0.2 * rnd(G, d, seed=9).float()
    ang = torch.arange(64, dtype=torch.float64)[:, None] * 50.0 ** (-2.0 * torch.arange(dims // 2, dtype=torch.float64) / dims)
    cos, sin = ang.cos().float().to(dev), ang.sin().float().to(dev)
    kc, vc = (torch.full((2, G, cap, D), 9.0, dtype=dtype, device=dev) for _ in range(2))
    S, n, m = torch.full((2, Hr, V, Nn), 7.0, **f), torch.full((2, 2, Hr, Nn), 7.0, **f), torch.full((2, 2, Hr), 7.0, **f)
    want, wq, wk = [], [], []
    for b in range(2):
        li = mcap * torch.tanh((gi[b] + ib).double() / mcap)
        lf = -oracle.softplus(-mcap * torch.tanh((gf[b] + fb).double() / mcap))
        want.append(oracle.mlstm_scan(q[b].double() * 0.4, k[b].double(), v[b].double(), li, lf).reshape(T, -1))
        real, pos = att[b, ..., :d].double(), torch.arange(T)
        wq.append(oracle.rotate(oracle.rms(real[:, :H].reshape(T, -1), eps, qw[:, :d].reshape(-1).double()).view(T, H, d), pos, dims, 50.0))
        wk.append(oracle.rotate(oracle.rms(real[:, H:H + G].reshape(T, -1), eps, kw[:, :d].reshape(-1).double()).view(T, G, d), pos, dims, 50.0))
    c0 = (H + 2 * G) * D
    a_dims = [0, H * D, (H + G) * D, H, G, D, H * d, G * d]
    m_dims = [c0, c0 + Hr * Nn, c0 + 2 * Hr * Nn, c0 + 2 * Hr * Nn + Hr * V, c0 + 2 * Hr * Nn + Hr * V + Hr, Hr, Nn, V]
    tol = 2e-5 if dtype == torch.float32 else 6e-3

    def step(rows, pos, live):
        return raw.parallel_step_(rows, a_dims, qw.to(dev).view(-1), kw.to(dev).view(-1), eps, cos, sin, kc, vc, m_dims,
                                  ib.to(dev), fb.to(dev), mcap, 0.4, S, n, m, pos, live)
    for t in range(T):
        live = torch.tensor([1, int(t < lens[1])], dtype=torch.int32, device=dev)
        pos = torch.full((2,), t, dtype=torch.int32, device=dev)
        rows = step_rows(dtype, dev, [att[:, t].reshape(2, -1), q[:, t].reshape(2, -1), k[:, t].reshape(2, -1),
                                      v[:, t].reshape(2, -1), gi[:, t], gf[:, t]])
        before = [x.clone() for x in (kc, vc, S, n, m)]
        step(rows[0] + 1, pos, torch.zeros(2, dtype=torch.int32, device=dev))
        assert all(torch.equal(x, y) for x, y in zip(before, (kc, vc, S, n, m)))
        qo, o = step(rows[t % 2], pos, live)
        for b in range(2):
            if t < lens[b]:
                assert N.rel_err(o[b:b + 1], want[b][t:t + 1]) < 10 * tol, (t, b)
                assert N.rel_err(qo[b, :, :d].reshape(1, -1), wq[b][t].reshape(1, -1)) < tol
                assert N.rel_err(kc[b, :, t % cap, :d].reshape(1, -1), wk[b][t].reshape(1, -1)) < tol
                assert torch.equal(vc[b, :, t % cap, :d].float().cpu(), att[b, t, H + G:, :d])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("B", [1, 2, 3, 4])
@pytest.mark.parametrize("width,ff,heads,v,vp", [(100, 192, 3, 20, 32), (640, 1344, 5, 64, 64), (2112, 4352, 8, 128, 128)])
def test_few_row_products(raw, dev, dtype, B, width, ff, heads, v, vp):
    """The weight-streaming products with their inputs and epilogues: norm, branch merge, gated unit, group norm with
    and without a gate, addition to the stream, two problems in a launch."""
    ld, eps, slots = -(-width // 64) * 64, 1e-3, heads * vp
    kp = -(-slots // 64) * 64
    if B * max(ld, kp, ff) * (4 if dtype == torch.float32 else 2) > 60000:
        pytest.skip("input rows do not fit the launch's LDS; the engine takes the GEMM path")

    def padded(t, n=ld):
        out = torch.zeros(*t.shape[:-1], n, dtype=t.dtype)
        out[..., :t.shape[-1]] = t
        return out
    x, a, b = (rnd(B, width, seed=s).float() for s in range(3))
    w, wa, wb = (1 + 0.3 * rnd(width, seed=10 + s).float() for s in range(3))
    X, A, Bb, W, WA, WB = (padded(t).to(dev) for t in (x, a, b, w, wa, wb))
    x, a, b, w, wa, wb = (t.double() for t in (x, a, b, w, wa, wb))
    tol = 3e-6 if dtype == torch.float32 else 8e-3
    M, Mr = typed(padded(rnd(104, width, seed=5, scale=width ** -0.5)), dtype, dev)
    normed = padded(oracle.rms(x, eps, w))
    y = raw.gemv_norm(X, W, width, eps, M, -1, None, None, None, None, None)
    assert y.dtype == torch.float32 and N.rel_err(y, normed @ Mr.T) < tol
    out = torch.empty_like(X)
    merged = x + 0.5 * (oracle.rms(a, eps, wa) + oracle.rms(b, eps, wb))
    U, Ur = typed(padded(rnd(2 * ff, width, seed=6, scale=width ** -0.5)), dtype, dev)
    g, u = (padded(oracle.rms(merged, eps, w)) @ Ur.T).chunk(2, -1)
    h = raw.gemv_norm(X, W, width, eps, U, 0, A, Bb, WA, WB, out)
    assert h.dtype == dtype and N.rel_err(out[:, :width], merged) < 1e-6 and N.rel_err(h, oracle.gelu_tanh(g) * u) < 2 * tol
    h, hr = typed(rnd(B, ff, seed=7), dtype, dev)
    Dn, Dr = typed(padded(rnd(ff, width, seed=8, scale=ff ** -0.5)).T.contiguous(), dtype, dev)
    Y = X.clone()
    raw.gemv_add_(Y, Dn, h)
    assert N.rel_err(Y[:, :width], x + (hr @ Dr.T)[:, :width]) < 2e-6
    o, nw = torch.zeros(B, heads, vp), torch.zeros(heads, vp)
    o[..., :v], nw[:, :v] = rnd(B, heads, v, seed=9).float(), 1 + 0.3 * rnd(heads, v, seed=13).float()
    G, Gr = typed(padded(rnd(heads * vp, width, seed=14, scale=slots ** -0.5)).T.contiguous(), dtype, dev)
    if kp > slots:
        z = torch.zeros(ld, kp - slots)
        G, Gr = torch.cat([G, z.to(dev, dtype)], 1).contiguous(), torch.cat([Gr, z.double()], 1)
    real, nr = o[..., :v].reshape(B, -1).double(), nw[:, :v].reshape(-1).double()
    for parts in {1, heads, 4 if heads * v % 4 == 0 else 1}:
        full = torch.zeros(B, heads, vp, dtype=torch.float64)
        full[..., :v] = oracle.rms(real, eps, nr, parts).view(B, heads, v)
        Y = X.clone()
        raw.gemv_group_add_(Y, G, o.to(dev).view(B, -1), nw.to(dev).view(-1), heads, v, vp, parts, eps)
        assert N.rel_err(Y[:, :width], x + (padded(full.view(B, -1), kp) @ Gr.T)[:, :width]) < tol
    gate = rnd(B, 16 + slots, seed=15).float()
    full = torch.zeros(B, heads, vp, dtype=torch.float64)
    full[..., :v] = oracle.rms(real, eps, nr, heads).view(B, heads, v)
    full = full.view(B, -1) * torch.sigmoid(gate[:, 16:].double())
    two = raw.gemv_branches(Dn, h, G, o.to(dev).view(B, -1), gate.to(dev), 16, nw.to(dev).view(-1), heads, v, vp, eps)
    assert N.rel_err(two[0, :, :width], (hr @ Dr.T)[:, :width]) < tol and N.rel_err(two[1, :, :width], (padded(full, kp) @ Gr.T)[:, :width]) < tol


@pytest.mark.parametrize("dtype", DTYPES)
def test_matrix_memory_extreme_gates(raw, dev, dtype):
    """A key written with a huge input gate long ago, forget gates at the cap: the maximum runs far from zero."""
    T, H, Nn, V = 190, 2, 32, 32
    q, qr = typed(rnd(T, H, Nn), dtype, dev)
    k, kr = typed(rnd(T, H, Nn, seed=1), dtype, dev)
    v, vr = typed(rnd(T, H, V, seed=2), dtype, dev)
    li, lf = torch.full((T, H), -14.0), torch.full((T, H), -3e-7)
    li[5] = 14.5
    lf[:, 1] = -14.9
    li[100:, 1] = 14.9
    want = oracle.mlstm_scan(qr, kr, vr, li.double(), lf.double())
    f = dict(device=dev, dtype=torch.float32)
    st = (torch.zeros(1, H, V, Nn, **f), torch.zeros(2, 1, H, Nn, **f), torch.zeros(2, 1, H, **f))
    rb = RowBatch(dev, False, seqs=pack([T]), scan_chunk=raw.scan_chunk(dtype == torch.float32))
    o = raw.scan_prefill_(q.view(T, -1), k.view(T, -1), v.view(T, -1), H, 1, Nn, V, 1.0, lf.to(dev), li.to(dev), None, None, *st,
                          rb.chunks, rb.scan_seqs)
    err = (o.cpu().double().view(T, H, V) - want).pow(2).mean(-1).sqrt() / want.pow(2).mean(-1).sqrt().clamp_min(1e-3)
    # (a token whose query is nearly orthogonal to the one stored key is ill-conditioned: 2e-4 in a plain 32-bit scan)
    assert float(err.max()) < (1e-3 if dtype == torch.float32 else 3e-2)
    assert float(err.median()) < (1e-6 if dtype == torch.float32 else 5e-3)


def prep(raw, dev, dtype, src, cfg, D, rb, cache, eps=1e-3, qw=None, kw=None, k_buf=None, v_buf=None, row_kv=None, keep=None):
    half = cfg["dims"] // 2
    f = cfg["base"] ** (-2.0 * torch.arange(half, dtype=torch.float64) / max(cfg["dims"], 1))
    a = torch.arange(4096, dtype=torch.float64)[:, None] * f
    cos, sin = a.cos().float().to(dev), a.sin().float().to(dev)
    H, G = cfg["H"], cfg["G"]
    return raw.attn_prep_(src, 0, H * D, (H + G) * D, qw, kw, H, G, D, H * cfg["d"], G * cfg["d"], eps, cos, sin, rb.slot, rb.pos,
                          row_kv, keep, k_buf, v_buf, *cache)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dims", [0, 12, 20])
def test_query_key_norm_and_rotation(raw, dev, dtype, dims):
    """Norm over all heads at once with the true width as divisor, rotation of the first dims, cache slots."""
    H, G, d, D, T, cap, eps = 6, 2, 20, 64, 9, 5, 1e-3
    cfg = {"H": H, "G": G, "d": d, "dims": dims, "base": 50.0}
    x = torch.zeros(T, H + 2 * G, D)
    x[..., :d] = rnd(T, H + 2 * G, d).float()
    xd, xr = typed(x, dtype, dev)
    qw, kw = torch.zeros(H, D), torch.zeros(G, D)
    qw[:, :d], kw[:, :d] = 1 + 0.2 * rnd(H, d, seed=3).float(), 1 + 0.2 * rnd(G, d, seed=4).float()
    rb = RowBatch(dev, False, seqs=[Sequence_(1, 0, T, 3)])
    k_buf, v_buf = (torch.zeros(T + 2, G, D, dtype=dtype, device=dev) for _ in range(2))
    cache = tuple(torch.full((2, G, cap, D), 9.0, dtype=dtype, device=dev) for _ in range(2))
    row_kv = torch.arange(2, T + 2, dtype=torch.int32, device=dev)
    keep = torch.tensor([int(p >= 10) for p in range(3, 3 + T)], dtype=torch.int32, device=dev)
    q = prep(raw, dev, dtype, xd.view(T, -1), cfg, D, rb, cache, eps, qw.to(dev).view(-1), kw.to(dev).view(-1), k_buf, v_buf, row_kv, keep)
    real = xr[..., :d]
    pos = torch.arange(3, 3 + T)
    wq = oracle.rotate(oracle.rms(real[:, :H].reshape(T, -1), eps, qw[:, :d].reshape(-1).double()).view(T, H, d), pos, dims, 50.0)
    wk = oracle.rotate(oracle.rms(real[:, H:H + G].reshape(T, -1), eps, kw[:, :d].reshape(-1).double()).view(T, G, d), pos, dims, 50.0)
    tol = 2e-6 if dtype == torch.float32 else 6e-3
    assert N.rel_err(q[..., :d].reshape(T, -1), wq.reshape(T, -1)) < tol and float(q[..., d:].float().abs().sum()) == 0
    assert N.rel_err(k_buf[2:, :, :d].reshape(T, -1), wk.reshape(T, -1)) < tol
    assert torch.equal(v_buf[2:].cpu(), xd.view(T, -1, D)[:, H + G:].cpu()) and float(k_buf[:2].float().abs().sum()) == 0
    for p in range(3, 3 + T):
        if p >= 10:
            assert torch.equal(cache[0][1, :, p % cap], k_buf[2 + p - 3]) and torch.equal(cache[1][1, :, p % cap], v_buf[2 + p - 3])
    assert float((cache[0][0].float() - 9).abs().sum()) == 0 and float((cache[0][1, :, 2:].float() - 9).abs().sum()) == 0


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,size", [(6, 2, 64, 13), (4, 4, 128, 64), (2, 1, 192, 65), (8, 2, 128, 300), (3, 1, 512, 40)])
def test_chunk_attention(raw, dev, dtype, H, G, D, size):
    """Both prefill kernels and the decode kernel, each against the oracle, on a pack of unequal sequences."""
    lens, scale = [1, size, size + 1, 2 * size + 7], 1.3 * D ** -0.5
    T = sum(lens)
    q, qr = typed(rnd(T, H, D), dtype, dev)
    k, kr = typed(rnd(T, G, D, seed=1), dtype, dev)
    v, vr = typed(rnd(T, G, D, seed=2), dtype, dev)
    rb = RowBatch(dev, False, seqs=pack(lens))
    runs, items, row_kv, keep, copies, kv_rows = rb.chunk_tables(size)
    assert copies is None and kv_rows == T and row_kv.tolist() == list(range(T))
    want = torch.cat([oracle.chunked_attention(qr[s.row0:s.row0 + s.rows], kr[s.row0:s.row0 + s.rows],
                                               vr[s.row0:s.row0 + s.rows], scale, size) for s in rb.seqs]).reshape(T, -1)
    tol = 5e-6 if dtype == torch.float32 else 8e-3
    assert N.rel_err(raw.attn_chunk(q, k, v, items, scale).view(T, -1), want) < tol
    if dtype == torch.bfloat16 and D <= 128:
        o = torch.zeros_like(q)
        for q0, n, key0, off, reps in runs:
            raw.attn_runs_(q, k, v, o, q0, n, key0, off, reps, scale)
        assert N.rel_err(o.view(T, -1), want) < tol
    # decode: the last token of every sequence from the cache of its chunk, all splits
    kc, vc = (torch.full((len(lens), G, size, D), 99.0, dtype=dtype, device=dev) for _ in range(2))
    for s in rb.seqs:
        for p in range((s.rows - 1) // size * size, s.rows):
            kc[s.slot, :, p % size], vc[s.slot, :, p % size] = k[s.row0 + p], v[s.row0 + p]
    last = torch.tensor([s.row0 + s.rows - 1 for s in rb.seqs], device=dev)
    pos = torch.tensor([n - 1 for n in lens], dtype=torch.int32, device=dev)
    for nsplit in (1, 4, 16):
        o = raw.attn_chunk_decode(q[last].contiguous(), kc, vc, pos, scale, nsplit)
        assert N.rel_err(o.view(len(lens), -1), want[last.cpu()]) < tol


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("size", [16, 64, 130, 400])
def test_attention_sees_exactly_its_chunk(raw, dev, dtype, size):
    """One key stands out.  Placed at the first position of the query's chunk it decides the output, one position
    earlier it does not exist; likewise one after the query."""
    H = G = 2
    D, T, scale = 64, 2 * size + 9, 0.5
    q, _ = typed(rnd(T, H, D), dtype, dev)
    k, _ = typed(0.1 * rnd(T, G, D, seed=1), dtype, dev)
    v, _ = typed(rnd(T, G, D, seed=2), dtype, dev)
    rb = RowBatch(dev, False, seqs=pack([T]))
    runs, items, *_ = rb.chunk_tables(size)
    for i in (size - 1, size, size + 5, 2 * size - 1, 2 * size, 2 * size + 8):
        lo = i // size * size
        for j, seen in ((lo, True), (i, True), (lo - 1, False), (i + 1, False)):
            if not 0 <= j < T or (j == i + 1 and j // size != i // size):
                continue
            k2 = k.clone()
            k2[j] = (q[i].float() * 2).to(dtype)            # score of about D: e^30 over the others
            outs = [raw.attn_chunk(q, k2, v, items, scale)[i]]
            if dtype == torch.bfloat16:
                o = torch.zeros_like(q)
                for q0, n, key0, off, reps in runs:
                    raw.attn_runs_(q, k2, v, o, q0, n, key0, off, reps, scale)
                outs.append(o[i])
            if j <= i:
                kc, vc = torch.zeros(1, G, size, D, dtype=dtype, device=dev), torch.zeros(1, G, size, D, dtype=dtype, device=dev)
                for p in range(lo, i + 1):
                    kc[0, :, p % size], vc[0, :, p % size] = k2[p], v[p]
                outs.append(raw.attn_chunk_decode(q[i:i + 1].contiguous(), kc, vc,
                                                  torch.tensor([i], dtype=torch.int32, device=dev), scale, 4)[0])
            for o in outs:
                near = float((o.float() - v[j].float()).abs().max())
                assert (near < 0.05) == seen, (i, j, near)


# ------------------------------------------------------------------ whole models
def forward(model, tokens, cuts=None, slot=0, batch=1):
    """Logits of every position, the prompt cut into portions of the given sizes (then single tokens)."""
    e = model.engine(max_len=1024, max_batch=batch)
    e.reset()
    out, at = [], 0
    for c in (cuts or [len(tokens)]):
        part = tokens[at:at + c]
        if len(part):
            out.append(e.extend([slot], [part], [range(len(part))]))
            at += len(part)
    while at < len(tokens):
        out.append(e.extend([slot], [tokens[at:at + 1]], [[0]]))
        at += 1
    return torch.cat(out)


SMALL = N.config([N.parallel(N.attention(size=9)), N.mamba(conv=4), N.parallel(N.attention(size=21), ff=None)], vocab=50, width=72)
ONE_KIND = [N.config([N.mamba(), N.mamba(ff=40)], width=40, vocab=31),
            N.config([N.parallel(N.attention(heads=1, kv_heads=1, dim=8, vdim=8, dims=8, size=1), N.memory(1, 8, 8, 1.0), 8)], width=8, vocab=9)]


@pytest.fixture(scope="module", params=DTYPES, ids=["f32", "bf16"])
def mixed(request, dev):
    return N.build(N.MIXED, request.param, dev)


@pytest.fixture(scope="module")
def mixed_want(mixed):
    t = N.prompt(150, 83, 3)
    return t, N.oracle_logits(mixed, t)


def test_layers_against_the_oracle(mixed):
    t = N.prompt(70, 83, 5)
    _, want = oracle.forward(mixed.config.raw, N.weights(mixed), t, keep_layers=True)
    got = mixed.engine(max_len=1024).layer_outputs(t)
    for i in range(len(want)):
        assert N.rel_err(got[i], want[i]) < MODEL_TOL[mixed.dtype], i


def test_prompt_whole_portions_and_decode(mixed, mixed_want):
    """The logits do not depend on how the prompt was cut: whole, two-token portions, chunk-sized and odd ones, and
    token by token through the decode step from the first."""
    t, want = mixed_want
    tol = MODEL_TOL[mixed.dtype]
    whole = forward(mixed, t)
    assert N.rel_err(whole, want) < tol
    for cuts in ([2] * 75, [64, 64, 22], [13, 29, 7, 101], [149], [1], [70, 1, 1, 2, 5]):
        assert N.rel_err(forward(mixed, t, cuts), want) < tol, cuts


@pytest.mark.parametrize("cfg", ONE_KIND + [SMALL])
@pytest.mark.parametrize("dtype", DTYPES)
def test_other_designs(dev, cfg, dtype):
    m = N.build(cfg, dtype, dev, seed=4)
    t = N.prompt(45, cfg["vocab"], 2)
    want = N.oracle_logits(m, t)
    assert N.rel_err(forward(m, t), want) < MODEL_TOL[dtype]
    assert N.rel_err(forward(m, t, [3]), want) < MODEL_TOL[dtype]


def test_batches_of_unequal_requests(mixed):
    """A pack of unequal prompts, then decoded together with some ending early and slots used again."""
    lens, extra = [1, 66, 17, 40], [12, 3, 12, 7]
    toks = [N.prompt(n + x, 83, 20 + i) for i, (n, x) in enumerate(zip(lens, extra))]
    want = [N.oracle_logits(mixed, t) for t in toks]
    e = mixed.engine(max_len=1024, max_batch=4)
    tol = MODEL_TOL[mixed.dtype]
    for slots in ([0, 1, 2, 3], [2, 0, 3, 1]):             # the second time in slots that others have used
        lg = e.extend(slots, [t[:n] for t, n in zip(toks, lens)], [[n - 1] for n in lens])
        for i in range(4):
            assert N.rel_err(lg[i:i + 1], want[i][lens[i] - 1:lens[i]]) < tol
        live = [0, 1, 2, 3]
        for s in range(max(extra)):
            gone = [i for i in live if s >= extra[i]]
            e.release([slots[i] for i in gone])
            live = [i for i in live if s < extra[i]]
            lg = e.extend([slots[i] for i in live], [toks[i][lens[i] + s:lens[i] + s + 1] for i in live], [[0]] * len(live))
            for r, i in enumerate(live):
                assert N.rel_err(lg[r:r + 1], want[i][lens[i] + s:lens[i] + s + 1]) < tol, (i, s)
        e.release([slots[i] for i in live])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", ["streamed", "blocks_too_wide", "gemm"])
def test_seven_streams_and_every_decode_path(dev, dtype, rows):
    """Decode steps of one and of seven sequences; of few sequences also where their rows do not fit the
    weight-streaming launch, block by block and altogether."""
    from eventgpt_amd.runtime.layered_engine import LayeredEngine
    m = N.build(N.MIXED, dtype, dev, seed=2)
    for B in ([7, 1] if rows == "streamed" else [3]):
        e = LayeredEngine(m, max_len=128, max_batch=B)
        if rows == "gemm":
            e.gemv_rows = 0
        if rows == "blocks_too_wide":
            for st in e.stages:
                st.block._lds = 0
        toks = [N.prompt(14 + 5 * i, 83, 70 + i) for i in range(B)]
        e.extend(list(range(B)), [t[:-6] for t in toks], [[]] * B)
        got = [e.extend(list(range(B)), [t[i:i + 1] if i < -1 else t[i:] for t in toks], [[0]] * B) for i in range(-6, 0)]
        for b, t in enumerate(toks):
            assert N.rel_err(torch.stack([g[b] for g in got]), N.oracle_logits(m, t)[-6:]) < MODEL_TOL[dtype], b


def test_long_prompts_run_in_portions(mixed, mixed_want):
    t, want = mixed_want
    e = mixed.engine(max_len=1024, max_batch=4)
    e.reset()
    e.PACK_ROWS = 60
    try:
        lg = e.extend([0, 2, 3], [t, t[:31], t[:100]], [range(150), [30], [99, 0]])
    finally:
        del e.PACK_ROWS
    tol = MODEL_TOL[mixed.dtype]
    assert N.rel_err(lg[:150], want) < tol and N.rel_err(lg[150:151], want[30:31]) < tol
    assert N.rel_err(lg[151:], want[[99, 0]]) < tol


def test_long_decoding(dev):
    """Several hundred steps over many chunk borders, in 32 bit: nothing drifts."""
    m = N.build(SMALL, torch.float32, dev, seed=6)
    t = N.prompt(420, 50, 8)
    want = N.oracle_logits(m, t)
    assert N.rel_err(forward(m, t, [3]), want) < MODEL_TOL[torch.float32]


def greedy(model, tokens, n):
    out = tokens.tolist()
    for _ in range(n):
        out.append(int(N.oracle_logits(model, torch.tensor(out))[-1].argmax()))
    return out[len(tokens):]


@pytest.fixture(scope="module")
def small(dev):
    return N.build(SMALL, torch.float32, dev, seed=9)


def test_greedy_generation(small):
    t = N.prompt(20, 50, 1)
    want = greedy(small, t, 24)
    assert small.generate(t[None], do_sample=False, max_new_tokens=24)[0].tolist() == want
    for graph in (False, True):                       # eager steps and several replays of one graph agree
        e = small.engine(max_len=4096)
        e.use_graph = graph
        for _ in range(3):
            assert e.generate(t, 24, eos_token_id=-1).tolist() == want
    stop = want[5]
    cut = want.index(stop) + 1
    assert small.generate(t, max_new_tokens=24, eos_token_id=stop)[0].tolist() == want[:cut]


def test_sampling_follows_the_distribution(small):
    t = N.prompt(20, 50, 1)
    one = small.generate(t, do_sample=True, temperature=1.0, top_k=1, max_new_tokens=8)[0].tolist()
    assert one == greedy(small, t, 8)
    g = [small.generate(t, do_sample=True, temperature=1.5, max_new_tokens=8,
                        generator=torch.Generator(device=small.device).manual_seed(s))[0].tolist() for s in (1, 1, 2)]
    assert g[0] == g[1] and g[0] != g[2] and all(0 <= x < 50 for x in g[0])


def test_teacher_forced_scores(small):
    t = N.prompt(30, 50, 4)
    e = small.engine(max_len=4096)
    got = e.score(t[:18], t[18:])
    assert N.rel_err(got, N.oracle_logits(small, t)[17:]) < MODEL_TOL[torch.float32]


def test_continuous_batching(small):
    """More requests than slots through the framework's scheduler: prompts join while others decode, slots are used
    again, every request gets the tokens it gets alone."""
    from eventgpt_amd.runtime.batcher import ContinuousBatcher
    from eventgpt_amd.runtime.layered_engine import LayeredEngine
    prompts = [N.prompt(n, 50, 40 + n) for n in (3, 1, 26, 11, 70, 5, 2)]
    budget = [9, 14, 4, 12, 6, 11, 8]
    b = ContinuousBatcher(LayeredEngine(small, max_len=256, max_batch=3, max_new_tokens=32), eos_token_id=-1, poll_every=2)
    reqs = [b.submit(p, n) for p, n in zip(prompts, budget)]
    b.run_until_idle()
    for r, p, n in zip(reqs, prompts, budget):
        assert r.tokens == greedy(small, p, n), r.rid


def test_command_line(small, tmp_path, capsys):
    from eventgpt_amd.cli.inference import run
    small.save_pretrained(str(tmp_path))
    t = N.prompt(12, 50, 30)
    got = run(["--model_path", str(tmp_path), "--token_ids", ",".join(map(str, t.tolist())), "--temperature", "0",
               "--max_new_tokens", "10", "--dtype", "float32", "--device", "cuda:0"])
    assert [int(x) for x in got.split(",")] == greedy(small, t, 10)


def test_trace_runner(small, tmp_path):
    """The trace program's steps, in process: a batch that starts together and ends request by request."""
    from eventgpt_amd.cli.trace_run import TraceRunner
    toks = {"x": N.prompt(30, 50, 60), "y": N.prompt(8, 50, 61)}
    want = {i: N.oracle_logits(small, t) for i, t in toks.items()}
    r = TraceRunner(small, 64)
    lg = r.step([{"id": "x", "tokens": toks["x"][:27].tolist(), "want": [26, 0]},
                 {"id": "y", "tokens": toks["y"][:7].tolist(), "want": []}], [])
    tol = MODEL_TOL[torch.float32]
    assert N.rel_err(lg, want["x"][[26, 0]]) < tol
    lg = r.step([{"id": "y", "tokens": toks["y"][7:].tolist(), "want": [0]},
                 {"id": "x", "tokens": toks["x"][27:28].tolist(), "want": [0]}], ["y"])
    assert N.rel_err(lg, torch.stack([want["y"][7], want["x"][27]])) < tol
    assert r.step([{"id": "x", "tokens": toks["x"][28:29].tolist(), "want": []}], []) is None
    lg = r.step([{"id": "x", "tokens": toks["x"][29:].tolist(), "want": [0]}], ["x"])
    assert N.rel_err(lg, want["x"][29:]) < tol and not r.slots


def test_limits_are_refused(small):
    e = small.engine(max_len=4096)
    e.reset()
    with pytest.raises(ValueError):
        e.prefill(torch.zeros(e.l_max + 1, dtype=torch.int32))
    with pytest.raises(ValueError):
        e.prefill(torch.zeros(0, dtype=torch.int32))
    bad = copy.deepcopy(SMALL)
    bad["layers"][0]["mixer"]["left"]["dim"] = 600
    with pytest.raises(ValueError):
        LayeredDecoder.from_config(LayeredConfig(bad), torch.bfloat16, small.device).engine(max_len=64)
