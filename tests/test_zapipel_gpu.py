"""Zapipel kernels and engine on the GPU against the plain oracle (tests/zapipel_oracle.py)."""
import copy

import pytest
import torch

import _zapipel as Z
import zapipel_oracle as oracle
from eventgpt_amd.models import LayeredConfig, LayeredDecoder
from eventgpt_amd.runtime import mixers
from eventgpt_amd.runtime.mixers import RowBatch, Sequence_

pytestmark = pytest.mark.gpu

F32, BF16 = torch.float32, torch.bfloat16
DTYPES = [F32, BF16]
MODEL_TOL = {F32: 1e-4, BF16: 8e-2}      # logits of a whole model, relative to their rms
GELU, SILU = 0, 1


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


def ints(dev, v):
    return torch.tensor(v, dtype=torch.int32, device=dev)


def padded(t, n):
    out = torch.zeros(*t.shape[:-1], n, dtype=t.dtype)
    out[..., :t.shape[-1]] = t
    return out


# ------------------------------------------------------------------ norms, logits
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [100, 64, 8200, 9000])
def test_layer_norms_around_a_sublayer(raw, dev, dtype, width):
    """Rows with a mean far from zero; slabs; picked and weighted rows; widths beyond what a thread keeps."""
    rows, ld, eps, f32 = 5, -(-width // 64) * 64, 3e-3, dtype == F32
    x, y, c = (rnd(rows, width, seed=s).float() + 20 * s for s in range(3))
    w, wy = (1 + 0.3 * rnd(width, seed=10 + s).float() for s in range(2))
    X, Y, C, W, WY = (padded(t, ld).to(dev) for t in (x, y, c, w, wy))
    x, y, c, w, wy = (t.double() for t in (x, y, c, w, wy))
    ln, tol = oracle.layer_norm, 2e-5 if f32 else 4e-3
    assert Z.rel_err(raw.norm_rows(X, ints(dev, [4, 0, 4]), W, width, eps, f32, True)[:, :width], ln(x, eps, w)[[4, 0, 4]]) < tol
    S = X.clone()
    xn = raw.add_norm_rows_(S, torch.stack([Y, C]), W, width, eps, f32, True)
    assert Z.rel_err(S[:, :width], x + y + c) < 1e-6 and Z.rel_err(xn[:, :width], ln(x + y + c, eps, w)) < tol
    for src, ref in ((Y, y), (torch.stack([Y, C]), y + c)):
        S = X.clone()
        xn = raw.post_norm_rows_(S, src, WY, W, width, eps, f32, True)
        want = x + ln(ref, eps, wy)
        assert Z.rel_err(S[:, :width], want) < 2e-6 and Z.rel_err(xn[:, :width], ln(want, eps, w)) < tol
        assert xn.dtype == dtype and float(xn[:, width:].float().abs().sum()) == 0 and float(S[:, width:].abs().sum()) == 0
    S = X.clone()
    raw.post_norm_rows_(S, Y, WY, None, width, eps, f32, False)              # RMS norm after, none before
    assert Z.rel_err(S[:, :width], x + oracle.rms(y, eps, wy)) < 2e-6
    pool, pr = typed(padded(rnd(9, width, seed=7), ld), dtype, dev)
    pick, f = [[8, 0], [3, 3], [1, 2], [7, 4], [5, 6]], torch.rand(rows, 2, generator=torch.Generator().manual_seed(1))
    mixed = (pr[torch.tensor(pick)] * f.double()[..., None]).sum(1)[:, :width]
    S = X.clone()
    xn = raw.mix_norm_rows_(S, pool, ints(dev, pick), f.to(dev), WY, W, width, eps, f32, True)
    want = x + ln(mixed, eps, wy)
    assert Z.rel_err(S[:, :width], want) < 2e-6 and Z.rel_err(xn[:, :width], ln(want, eps, w)) < tol
    S = X.clone()
    raw.mix_norm_rows_(S, pool, ints(dev, pick), f.to(dev), None, None, width, eps, f32, True)
    assert Z.rel_err(S[:, :width], x + mixed) < 1e-6


def test_capped_logits(raw, dev):
    x = (rnd(7, 96) * 30).float()
    for scale, cap in ((0.7, 4.0), (3.0, 50.0), (0.25, 0.0)):
        y = x.clone().to(dev)
        raw.cap_logits_(y, scale, cap)
        want = oracle.softcap(x.double(), scale, cap) if cap else x.double() * scale
        assert torch.allclose(y.cpu().double(), want, rtol=2e-6, atol=1e-6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("B", [1, 2, 3, 4])
@pytest.mark.parametrize("width,n", [(100, 40), (640, 200), (4200, 33)])
def test_few_row_products(raw, dev, dtype, B, width, n):
    """The weight-streaming products behind a layer norm, behind the norm of a sublayer's output, behind the RMS norm of some
    columns (with the latents stored by the same launch), and plain."""
    ld, eps = -(-width // 64) * 64, 1e-3
    if B * ld * (4 if dtype == F32 else 2) > 60000:
        pytest.skip("input rows do not fit the launch's LDS; the engine takes the GEMM path")
    x, a = (rnd(B, width, seed=s).float() + 3 * s for s in range(2))
    w, wa = (1 + 0.3 * rnd(width, seed=10 + s).float() for s in range(2))
    X, A, W, WA = (padded(t, ld).to(dev) for t in (x, a, w, wa))
    x, a, w, wa = (t.double() for t in (x, a, w, wa))
    tol = 5e-6 if dtype == F32 else 8e-3
    M, Mr = typed(padded(rnd(104, width, seed=5, scale=width ** -0.5), ld), dtype, dev)
    ln = oracle.layer_norm
    xn = torch.empty(B, ld, dtype=dtype, device=dev)
    y = raw.gemv_norm(X, W, width, eps, M, -1, None, None, None, None, None, True, xn)
    assert Z.rel_err(y, padded(ln(x, eps, w), ld) @ Mr.T) < tol and Z.rel_err(xn, padded(ln(x, eps, w), ld)) < tol
    out, new = torch.empty_like(X), x + ln(a, eps, wa)
    y = raw.gemv_norm(X, W, width, eps, M, -1, A, None, WA, None, out, True, xn, 0.6, 2.0)
    want = padded(ln(new, eps, w), ld)
    assert Z.rel_err(out[:, :width], new) < 2e-6 and Z.rel_err(xn, want) < tol
    assert Z.rel_err(y, oracle.softcap(want @ Mr.T, 0.6, 2.0)) < tol
    g, u = (want @ Mr.T).chunk(2, -1)
    h = raw.gemv_norm(X, W, width, eps, M, SILU, A, None, WA, None, torch.empty_like(X), True)
    assert h.dtype == dtype and Z.rel_err(h, oracle.silu(g) * u) < 2 * tol
    # columns of a projection: 24 others, n for the product, then 21 latents
    Q, R = -(-n // 64) * 64, 64
    src, sr = typed(rnd(2, B, 24 + Q + 24, seed=6), F32, dev)
    sr = sr.sum(0)
    qw, cw = 1 + 0.2 * rnd(n, seed=8).float(), 1 + 0.2 * rnd(21, seed=9).float()
    P, Pr = typed(padded(rnd(136, n, seed=11, scale=n ** -0.5), Q), dtype, dev)
    cache = torch.full((B, 5, R), 7.0, dtype=dtype, device=dev)
    pos, live = [4, 0, 2, 3][:B], [1, 1, 0, 1][:B]
    y = raw.gemv_rows(src, 24, n, padded(qw, Q).to(dev), eps, P, 24 + Q, 21, padded(cw, R).to(dev), cache, ints(dev, pos), ints(dev, live))
    assert Z.rel_err(y, padded(oracle.rms(sr[:, 24:24 + n], eps, qw.double()), Q) @ Pr.T) < tol
    lat = oracle.rms(sr[:, 24 + Q:24 + Q + 21], eps, cw.double())
    for b in range(B):
        rest = [p for p in range(5) if p != pos[b] or not live[b]]
        assert float((cache[b, rest].float() - 7).abs().max()) == 0
        if live[b]:
            assert Z.rel_err(cache[b, pos[b]:pos[b] + 1], padded(lat[b:b + 1], R)) < (1e-6 if dtype == F32 else 4e-3)
    assert torch.equal(y, raw.gemv_rows(src, 24, n, padded(qw, Q).to(dev), eps, P, 0, 0, None, None, None, None))
    h, hr = typed(rnd(B, Q, seed=12), dtype, dev)
    assert Z.rel_err(raw.gemv_plain(P, h), hr @ Pr.T) < 2e-6


# ------------------------------------------------------------------ latent attention
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("nq,nc", [(24, 40), (9, 100), (600, 512)])
def test_latents_go_to_their_places(raw, dev, dtype, nq, nc):
    """Norm over the true columns, query rows out, latents into the right slot and position and nowhere else."""
    M, Q, R, eps = 6, -(-nq // 64) * 64, mixers.pad_latent(nc), 1e-3
    src, sr = typed(rnd(M, Q + R + 8), dtype, dev)
    qw, cw = 1 + 0.2 * rnd(nq, seed=1).float(), 1 + 0.2 * rnd(nc, seed=2).float()
    cache = torch.full((3, 7, R), 5.0, dtype=dtype, device=dev)
    slot, pos = [2, 2, 2, 0, 0, 2], [4, 5, 6, 0, 1, 0]
    q = raw.latent_prep_(src, 0, nq, padded(qw, Q).to(dev), Q, nc, padded(cw, R).to(dev), cache, ints(dev, slot), ints(dev, pos), None, eps, dtype == F32)
    tol = 1e-6 if dtype == F32 else 4e-3
    assert Z.rel_err(q, padded(oracle.rms(sr[:, :nq], eps, qw.double()), Q)) < tol
    lat = padded(oracle.rms(sr[:, Q:Q + nc], eps, cw.double()), R)
    for i in range(M):
        assert Z.rel_err(cache[slot[i], pos[i]][None], lat[i:i + 1]) < tol
    used = set(zip(slot, pos))
    assert all(float((cache[s, p].float() - 5).abs().max()) == 0 for s in range(3) for p in range(7) if (s, p) not in used)
    buf = raw.latent_gather(cache, ints(dev, [[2, 0, 0, 7], [0, 0, 7, 2]]), 9)
    assert torch.equal(buf, torch.cat([cache[2], cache[0, :2]]))
    # nothing but the queries (a layer that reads another one's latents), and rows that are slabs
    two = torch.stack([src.float() * 0.5, src.float() * 0.5])
    q2 = raw.latent_prep_(two, 0, nq, padded(qw, Q).to(dev), 0, 0, None, None, None, ints(dev, pos), None, eps, dtype == F32)
    assert Z.rel_err(q2, q) < tol
    kept = cache.clone()
    raw.latent_prep_(two[:, :3], 0, nq, None, Q, nc, padded(cw, R).to(dev), cache, None, ints(dev, [1, 2, 3]), ints(dev, [0, 0, 0]), eps, dtype == F32)
    assert torch.equal(kept, cache)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,N,K", [(5, 64, 64), (20, 512, 128), (3, 128, 384), (1, 64, 512)])
def test_products_per_head(raw, dev, dtype, H, N, K):
    w, wr = typed(rnd(H, N, K, scale=K ** -0.5), dtype, dev)
    tol = 2e-6 if dtype == F32 else 6e-3
    for M in (1, 3, 16, 17, 40, 300):
        x, xr = typed(rnd(M, H * K, seed=M), dtype, dev)
        gate, gr = typed(rnd(M, 16 + H + (-H) % 8, seed=M + 1), dtype, dev)
        want = (wr[None] @ xr.view(M, H, K, 1))[..., 0]
        assert Z.rel_err(raw.head_linear(x, w, None, 0), want) < tol
        gated = want * torch.sigmoid(gr[:, 11:11 + H, None])
        assert Z.rel_err(raw.head_linear(x, w, gate, 11), gated) < tol
        half = x.float() * 0.5                       # fp32 slabs that sum to x
        assert Z.rel_err(raw.head_linear(torch.stack([half, half]), w, gate, 11), gated) < tol


def latent_want(q, c, wv, g, scale):
    """One query ``[H, R]`` over latents ``[n, R]``: the attended latent per head, out through ``wv [H, D, R]``, gated."""
    s = (c @ q.T) * scale
    p = torch.softmax(s, 0)
    return (wv @ (p.T @ c)[..., None])[..., 0] * torch.sigmoid(g)[:, None]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,R", [(1, 64), (6, 128), (16, 256), (18, 384), (40, 512)])
def test_attention_over_latents(raw, dev, dtype, H, R):
    """Every length around the edges of the key tiles and splits, in a shuffled set of slots, any number of splits."""
    lens = [1, 2, 31, 32, 33, 63, 64, 65, 127, 128, 129, 255, 256, 257, 500, 700]
    B, cap, D, scale = len(lens), 700, 64, 1.7 * R ** -0.5
    c, cr = typed(rnd(B, cap, R), dtype, dev)
    q, qr = typed(rnd(B, H, R, seed=1), dtype, dev)
    wv, wr = typed(rnd(H, D, R, seed=2, scale=R ** -0.5), dtype, dev)
    gate, gr = typed(rnd(B, H + (-H) % 8, seed=3), dtype, dev)
    slots = [(5 * i + 3) % B for i in range(B)]
    want = torch.stack([latent_want(qr[b], cr[slots[b], :lens[b]], wr, gr[b, :H], scale) for b in range(B)])
    # what lies behind a sequence's end is an earlier owner's
    for b in range(B):
        c[slots[b], lens[b]:] = 50.0
    pos = ints(dev, [n - 1 for n in lens])
    tol = 1e-5 if dtype == F32 else 1e-2
    for nsplit in (1, 2, 3, 7, 64):
        o = raw.latent_attend(q, c, ints(dev, slots), pos, scale, nsplit, wv, gate, 0)
        assert Z.rel_err(o.view(B, -1), want.view(B, -1)) < tol, nsplit
    o = raw.latent_attend(q[:3].contiguous(), c, None, ints(dev, [4, 0, 250]), scale, 4, wv, gate[:3], 0)
    for b, n in enumerate((5, 1, 251)):
        assert Z.rel_err(o[b].reshape(1, -1), latent_want(qr[b], c[b, :n].cpu().double(), wr, gr[b, :H], scale).reshape(1, -1)) < tol


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("R", [64, 128, 512])
def test_a_far_latent_is_found(raw, dev, dtype, R):
    """One latent stands out for one head.  Anywhere among the visible positions it decides that head's output, one past
    the query's position it does not exist."""
    H, cap, scale = 17, 900, 0.25
    q, _ = typed(rnd(1, H, R), dtype, dev)
    base, _ = typed(0.05 * rnd(1, cap, R, seed=1), dtype, dev)
    wv, wr = typed(rnd(H, 64, R, seed=2, scale=R ** -0.5), dtype, dev)
    gate = torch.full((1, 24), 30.0, dtype=dtype, device=dev)
    for head in (0, 15, 16):
        loud = (q[0, head].float() * (240.0 / R)).to(dtype)      # its score: about 60
        for i in (0, 31, 64, 127, 128, 300, 899):
            for j in sorted({0, i // 2, max(i - 1, 0), i, i + 1}):
                if j >= cap:
                    continue
                c = base.clone()
                c[0, j] = loud
                for nsplit in (1, 8):
                    o = raw.latent_attend(q, c, None, ints(dev, [i]), scale, nsplit, wv, gate, 0)[0, head].double().cpu()
                    alone = (wr[head] @ loud.double().cpu())
                    near = float((o - alone).abs().max() / alone.abs().max())
                    assert (near < 0.02) == (j <= i), (head, i, j, near)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,D", [(3, 64), (4, 128), (2, 192)])
def test_expanded_attention_with_gates(raw, dev, dtype, H, D):
    """The prompt kernels on keys and values that are columns of one matrix, heads gated, a pack of whole sequences and of
    one that goes on after cached keys."""
    seqs, row = [], 0
    for slot, (start, n) in enumerate([(0, 1), (0, 70), (333, 300), (64, 2), (0, 600)]):
        seqs.append(Sequence_(slot, row, n, start))
        row += n
    rb = RowBatch(dev, False, seqs=seqs)
    runs, items, _, kv_rows = rb.causal_tables()
    q, qr = typed(rnd(row, H, D), dtype, dev)
    kv, kvr = typed(rnd(kv_rows, 2 * H * D, seed=1), dtype, dev)
    src, sr = typed(rnd(row, 8 + H + (-H) % 8, seed=2), dtype, dev)
    k, v = kv[:, :H * D].unflatten(1, (H, D)), kv[:, H * D:].unflatten(1, (H, D))
    kr, vr = kvr[:, :H * D].unflatten(1, (H, D)), kvr[:, H * D:].unflatten(1, (H, D))
    scale, want = 1.4 * D ** -0.5, torch.zeros(row, H, D, dtype=torch.float64)
    for s, (_, _, key0, off, _) in zip(seqs, runs):
        n = off + s.rows
        qq = torch.cat([torch.zeros(off, H, D, dtype=torch.float64), qr[s.row0:s.row0 + s.rows]])
        a = (qq.transpose(0, 1) @ kr[key0:key0 + n].permute(1, 2, 0)) * scale
        a = torch.softmax(a + torch.full((n, n), float("-inf"), dtype=torch.float64).triu(1), -1) @ vr[key0:key0 + n].transpose(0, 1)
        want[s.row0:s.row0 + s.rows] = a.transpose(0, 1)[off:]
    want = (want * torch.sigmoid(sr[:, 8:8 + H, None])).view(row, -1)
    tol = 1e-5 if dtype == F32 else 8e-3
    assert Z.row_err(raw.attn_chunk(q, k, v, items, scale, src, 8).view(row, -1), want) < tol
    if dtype == BF16 and D <= 128:
        o = torch.zeros_like(q)
        for q0, n, key0, off, reps in runs:
            raw.attn_runs_(q, k, v, o, q0, n, key0, off, reps, scale, src, 8)
        assert Z.row_err(o.view(row, -1), want) < tol


# ------------------------------------------------------------------ experts
@pytest.mark.parametrize("E,top", [(1, 1), (5, 3), (8, 8), (64, 6), (70, 1), (200, 40)])
def test_routing(raw, dev, E, top):
    M, ld = 37, -(-E // 8) * 8
    z, b = rnd(M, ld).float(), rnd(E, seed=1).float()
    z[3, :E] = b.neg() + 2                            # all equal: the first ones
    z[4, E - 1] = 40
    idx, w = raw.moe_route(z.to(dev), b.to(dev), top)
    both = (z[:, :E] + b).double()
    which, want = oracle.route(both, top)
    keep = torch.ones(M, dtype=torch.bool)
    keep[3] = False                                   # (the sums are equal up to rounding only)
    assert torch.equal(idx.cpu().long()[keep], which[keep]) and torch.allclose(w.cpu().double(), want, rtol=1e-5, atol=1e-7)
    assert sorted(set(idx[3].tolist())) == sorted(idx[3].tolist())
    z[:] = 0.5
    z[5] = float("nan")
    z[6] = float("-inf")
    idx, w = raw.moe_route(torch.stack([z, z]).to(dev), torch.zeros(E, device=dev), top)      # slabs; ties; no number at all
    assert idx[0].tolist() == list(range(top)) and torch.allclose(w[0].cpu(), torch.full((top,), 1.0 / top))
    assert int(idx.min()) >= 0 and int(idx.max()) < E and all(len(set(r)) == top for r in idx.tolist())


@pytest.mark.parametrize("M,E,top", [(1, 1, 1), (5, 9, 2), (700, 6, 3), (3000, 70, 4), (64, 5, 5)])
def test_sorting_by_expert(raw, dev, M, E, top):
    g = torch.Generator().manual_seed(M)
    idx = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(M)])
    if E > 4:
        idx[idx == 2] = 3 if top == 1 else 2          # (an expert that nobody chooses)
    for t in (idx, torch.zeros_like(idx), torch.full_like(idx, E - 1)):
        perm, inv, start = (x.cpu().long() for x in raw.moe_group(t.to(dev, torch.int32), E))
        flat = t.reshape(-1)
        assert torch.equal(perm, torch.sort(flat, stable=True).indices) and torch.equal(inv.view(-1)[perm], torch.arange(M * top))
        assert torch.equal(start, torch.cat([torch.zeros(1, dtype=torch.long), torch.bincount(flat, minlength=E).cumsum(0)]))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("counts,K,N", [([1], 192, 320), ([3, 0, 7, 0, 1], 192, 320), ([33, 64, 0, 65, 20], 192, 320),
                                        ([100, 1, 130, 90], 192, 320), ([300, 129, 0, 500, 128, 255], 192, 320),
                                        ([1300, 257, 0, 1600], 192, 320), ([1800, 1500], 64, 4736)])
def test_grouped_products(raw, dev, dtype, counts, K, N):
    """Every tile size (by the average group), more tiles than workgroups, empty and uneven groups, gathered and consecutive
    rows, all activations."""
    E, top = len(counts), 2
    rows = sum(counts)
    M = -(-rows // top)
    counts = counts[:-1] + [counts[-1] + M * top - rows]
    rows = M * top
    start = torch.tensor([0] + counts).cumsum(0)
    perm = torch.randperm(rows, generator=torch.Generator().manual_seed(rows))
    x, xr = typed(rnd(M, K), dtype, dev)
    w, wr = typed(rnd(E, N, K, seed=1, scale=K ** -0.5), dtype, dev)
    st, pm = start.to(dev, torch.int32), perm.to(dev, torch.int32)

    def grouped(a):
        return torch.cat([a[start[e]:start[e + 1]] @ wr[e].T for e in range(E)])
    y = grouped(xr[perm // top])
    tol = 2e-6 if dtype == F32 else 8e-3
    assert Z.rel_err(raw.moe_linear(x, w, st, pm, top, -1), y) < tol
    g, u = y.chunk(2, -1)
    assert Z.rel_err(raw.moe_linear(x, w, st, pm, top, SILU), oracle.silu(g) * u) < 2 * tol
    gelu = torch.nn.functional.gelu(g, approximate="tanh")
    assert Z.rel_err(raw.moe_linear(x, w, st, pm, top, GELU), gelu * u) < 2 * tol
    full, fr = typed(rnd(rows, K, seed=2), dtype, dev)
    assert Z.rel_err(raw.moe_linear(full, w, st, None, 1, -1), grouped(fr)) < tol


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("E,top,K,ff,N", [(1, 1, 64, 64, 64), (5, 3, 128, 64, 192), (9, 2, 2112, 704, 2112), (70, 8, 64, 128, 64)])
def test_experts_of_a_few_rows(raw, dev, dtype, E, top, K, ff, N):
    wg, wgr = typed(rnd(E, 2 * ff, K, scale=K ** -0.5), dtype, dev)
    wd, wdr = typed(rnd(E, N, ff, seed=1, scale=ff ** -0.5), dtype, dev)
    bias = rnd(E, seed=3).float()
    for B in (1, 2, 4):
        x, xr = typed(rnd(B, K, seed=10 + B), dtype, dev)
        z = padded(rnd(B, E, seed=20 + B).float(), -(-E // 8) * 8)
        which, f = oracle.route((z[:, :E] + bias).double(), top)
        want = torch.zeros(B, N, dtype=torch.float64)
        for b in range(B):
            for e, fe in zip(which[b].tolist(), f[b]):
                g, u = (wgr[e] @ xr[b]).chunk(2)
                want[b] += fe * (wdr[e] @ (oracle.silu(g) * u))
        got = raw.moe_step(x, z.to(dev), bias.to(dev), top, wg, wd, SILU)
        assert Z.rel_err(got, want) < (3e-6 if dtype == F32 else 1e-2)


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


CASES = [(Z.MIXED, F32), (Z.all_chosen(Z.MIXED), BF16), (Z.WIDE, F32), (Z.WIDE, BF16)]


@pytest.fixture(scope="module", params=CASES, ids=["mixed-f32", "mixed-bf16", "wide-f32", "wide-bf16"])
def model(request, dev):
    return Z.build(*request.param, dev)


@pytest.fixture(scope="module")
def want150(model):
    t = Z.prompt(150, model.config.vocab_size, 3)
    return t, Z.oracle_logits(model, t)


def test_layers_against_the_oracle(model):
    t = Z.prompt(70, model.config.vocab_size, 5)
    _, want = oracle.forward(model.config.raw, Z.weights(model), t, keep_layers=True)
    got = model.engine(max_len=1024).layer_outputs(t)
    for i in range(len(want)):
        assert Z.rel_err(got[i], want[i]) < MODEL_TOL[model.dtype], i


def test_prompt_whole_portions_and_decode(model, want150):
    """The logits do not depend on how the prompt was cut: whole, portions of two tokens, odd ones, and token by token
    through the decode step from the first."""
    t, want = want150
    tol = MODEL_TOL[model.dtype]
    for cuts in (None, [2] * 75, [64, 64, 22], [13, 29, 7, 101], [149], [1], [70, 1, 1, 2, 5]):
        assert Z.rel_err(forward(model, t, cuts), want) < tol, cuts


@pytest.mark.parametrize("over_cache", [False, True])
def test_portions_both_ways(model, want150, monkeypatch, over_cache):
    """A portion's attention, with its keys expanded and over the cached latents."""
    t, want = want150
    monkeypatch.setattr(mixers.LatentAttentionMixer, "absorbs", lambda self, rows: over_cache)
    for cuts in ([2] * 75, [100, 50], [31, 33, 86]):
        assert Z.rel_err(forward(model, t, cuts), want) < MODEL_TOL[model.dtype], cuts


def test_batches_of_unequal_requests(model):
    """A pack of unequal prompts, then decoded together with some ending early and slots used again."""
    V = model.config.vocab_size
    lens, extra = [1, 66, 17, 40], [12, 3, 12, 7]
    toks = [Z.prompt(n + x, V, 20 + i) for i, (n, x) in enumerate(zip(lens, extra))]
    want = [Z.oracle_logits(model, t) for t in toks]
    e = model.engine(max_len=1024, max_batch=4)
    tol = MODEL_TOL[model.dtype]
    for slots in ([0, 1, 2, 3], [2, 0, 3, 1]):             # the second time in slots that others have used
        lg = e.extend(slots, [t[:n] for t, n in zip(toks, lens)], [[n - 1] for n in lens])
        for i in range(4):
            assert Z.rel_err(lg[i:i + 1], want[i][lens[i] - 1:lens[i]]) < tol
        live = [0, 1, 2, 3]
        for s in range(max(extra)):
            gone = [i for i in live if s >= extra[i]]
            e.release([slots[i] for i in gone])
            live = [i for i in live if s < extra[i]]
            lg = e.extend([slots[i] for i in live], [toks[i][lens[i] + s:lens[i] + s + 1] for i in live], [[0]] * len(live))
            for r, i in enumerate(live):
                assert Z.rel_err(lg[r:r + 1], want[i][lens[i] + s:lens[i] + s + 1]) < tol, (i, s)
        e.release([slots[i] for i in live])


def test_a_waiting_request_is_left_alone(model):
    """A sequence that sits out steps of another one, and portions of two sequences in one pack, one over cached tokens."""
    V, tol = model.config.vocab_size, MODEL_TOL[model.dtype]
    a, b = Z.prompt(60, V, 31), Z.prompt(90, V, 32)
    wa, wb = Z.oracle_logits(model, a), Z.oracle_logits(model, b)
    e = model.engine(max_len=1024, max_batch=4)
    e.reset()
    e.extend([1, 3], [a[:20], b[:33]], [[], []])
    for i in range(20, 26):
        assert Z.rel_err(e.extend([1], [a[i:i + 1]], [[0]]), wa[i:i + 1]) < tol
    lg = e.extend([3, 1], [b[33:70], a[26:28]], [range(37), [0, 1]])
    assert Z.rel_err(lg, torch.cat([wb[33:70], wa[26:28]])) < tol
    lg = e.extend([3, 1], [b[70:71], a[28:29]], [[0], [0]])
    assert Z.rel_err(lg, torch.cat([wb[70:71], wa[28:29]])) < tol


@pytest.mark.parametrize("cfg,dtype", CASES[:2])
@pytest.mark.parametrize("rows", ["streamed", "blocks_too_wide", "gemm"])
def test_seven_streams_and_every_decode_path(dev, cfg, dtype, rows):
    """Decode steps of one and of seven sequences; of few sequences also where their rows do not fit the
    weight-streaming launch, block by block and altogether."""
    from eventgpt_amd.runtime.layered_engine import LayeredEngine
    m = Z.build(cfg, dtype, dev, seed=2)
    for B in ([7, 1] if rows == "streamed" else [3]):
        e = LayeredEngine(m, max_len=128, max_batch=B)
        if rows == "gemm":
            e.gemv_rows = 0
        if rows == "blocks_too_wide":
            for st in e.stages:
                st.block._lds = 0
        toks = [Z.prompt(14 + 5 * i, 83, 70 + i) for i in range(B)]
        e.extend(list(range(B)), [t[:-6] for t in toks], [[]] * B)
        got = [e.extend(list(range(B)), [t[i:i + 1] if i < -1 else t[i:] for t in toks], [[0]] * B) for i in range(-6, 0)]
        for b, t in enumerate(toks):
            assert Z.rel_err(torch.stack([g[b] for g in got]), Z.oracle_logits(m, t)[-6:]) < MODEL_TOL[dtype], b


def test_chosen_experts_in_16_bits(dev):
    """A router's choice can turn on rounding where two logits are close; everywhere else 16 bits choose the same."""
    m = Z.build(Z.MIXED, BF16, dev, seed=4)
    t = Z.prompt(120, 83, 6)
    margins, plain = [], oracle.route

    def watched(z, top):
        if top < z.shape[1]:
            s = torch.sort(z, dim=-1, descending=True).values
            margins.append(s[:, top - 1] - s[:, top])
        return plain(z, top)
    oracle.route = watched
    try:
        want = Z.oracle_logits(m, t)
    finally:
        oracle.route = plain
    clear = torch.stack(margins).min(0).values > 0.1
    assert int(clear.sum()) > 40
    for cuts in (None, [60, 30, 2], [110]):
        got = forward(m, t, cuts).cpu().double()
        err = (got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()
        assert float(err[clear].max()) < 2 * MODEL_TOL[BF16] and float(err.median()) < MODEL_TOL[BF16] / 2


def test_long_prompts_run_in_portions(model, want150):
    t, want = want150
    e = model.engine(max_len=1024, max_batch=4)
    e.reset()
    e.PACK_ROWS = 60
    try:
        lg = e.extend([0, 2, 3], [t, t[:31], t[:100]], [range(150), [30], [99, 0]])
    finally:
        del e.PACK_ROWS
    tol = MODEL_TOL[model.dtype]
    assert Z.rel_err(lg[:150], want) < tol and Z.rel_err(lg[150:151], want[30:31]) < tol
    assert Z.rel_err(lg[151:], want[[99, 0]]) < tol


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_prompt_and_long_decoding(dev, dtype):
    """Hundreds of tokens in a prompt (the flash kernels), then hundreds of steps: nothing drifts; the cache is filled to its
    last position."""
    from eventgpt_amd.runtime.layered_engine import LayeredEngine
    m = Z.build(Z.all_chosen(Z.SMALL), dtype, dev, seed=6)
    t = Z.prompt(700, 50, 8)
    want = Z.oracle_logits(m, t)
    tol = MODEL_TOL[dtype]
    for first in (400, 3):
        e = LayeredEngine(m, max_len=700, max_batch=2)
        got = [e.extend([1], [t[:first]], [range(first)])]
        got += [e.extend([1], [t[i:i + 1]], [[0]]) for i in range(first, 700)]
        assert Z.rel_err(torch.cat(got), want) < tol
        with pytest.raises(ValueError):
            e.extend([1], [t[:1]], [[]])


def greedy(model, tokens, n):
    out = tokens.tolist()
    for _ in range(n):
        out.append(int(Z.oracle_logits(model, torch.tensor(out))[-1].argmax()))
    return out[len(tokens):]


@pytest.fixture(scope="module")
def small(dev):
    return Z.build(Z.SMALL, F32, dev, seed=9)


def test_greedy_generation(small):
    t = Z.prompt(20, 50, 1)
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
    t = Z.prompt(20, 50, 1)
    one = small.generate(t, do_sample=True, temperature=1.0, top_k=1, max_new_tokens=8)[0].tolist()
    assert one == greedy(small, t, 8)
    g = [small.generate(t, do_sample=True, temperature=1.5, max_new_tokens=8,
                        generator=torch.Generator(device=small.device).manual_seed(s))[0].tolist() for s in (1, 1, 2)]
    assert g[0] == g[1] and g[0] != g[2] and all(0 <= x < 50 for x in g[0])


def test_teacher_forced_scores(small):
    t = Z.prompt(30, 50, 4)
    got = small.engine(max_len=4096).score(t[:18], t[18:])
    assert Z.rel_err(got, Z.oracle_logits(small, t)[17:]) < MODEL_TOL[F32]


def test_continuous_batching(small):
    """More requests than slots through the framework's scheduler: prompts join while others decode, slots are used
    again, every request gets the tokens it gets alone."""
    from eventgpt_amd.runtime.batcher import ContinuousBatcher
    from eventgpt_amd.runtime.layered_engine import LayeredEngine
    prompts = [Z.prompt(n, 50, 40 + n) for n in (3, 1, 26, 11, 70, 5, 2)]
    budget = [9, 14, 4, 12, 6, 11, 8]
    b = ContinuousBatcher(LayeredEngine(small, max_len=256, max_batch=3, max_new_tokens=32), eos_token_id=-1, poll_every=2)
    reqs = [b.submit(p, n) for p, n in zip(prompts, budget)]
    b.run_until_idle()
    for r, p, n in zip(reqs, prompts, budget):
        assert r.tokens == greedy(small, p, n), r.rid


def test_command_line(small, tmp_path):
    from eventgpt_amd.cli.inference import run
    small.save_pretrained(str(tmp_path))
    t = Z.prompt(12, 50, 30)
    got = run(["--model_path", str(tmp_path), "--token_ids", ",".join(map(str, t.tolist())), "--temperature", "0",
               "--max_new_tokens", "10", "--dtype", "float32", "--device", "cuda:0"])
    assert [int(x) for x in got.split(",")] == greedy(small, t, 10)


def test_trace_runner(small):
    """The trace program's steps, in process: a batch that starts together and ends request by request."""
    from eventgpt_amd.cli.trace_run import TraceRunner
    toks = {"x": Z.prompt(30, 50, 60), "y": Z.prompt(8, 50, 61)}
    want = {i: Z.oracle_logits(small, t) for i, t in toks.items()}
    r = TraceRunner(small, 64)
    lg = r.step([{"id": "x", "tokens": toks["x"][:27].tolist(), "want": [26, 0]},
                 {"id": "y", "tokens": toks["y"][:7].tolist(), "want": []}], [])
    tol = MODEL_TOL[F32]
    assert Z.rel_err(lg, want["x"][[26, 0]]) < tol
    lg = r.step([{"id": "y", "tokens": toks["y"][7:].tolist(), "want": [0]},
                 {"id": "x", "tokens": toks["x"][27:28].tolist(), "want": [0]}], ["y"])
    assert Z.rel_err(lg, torch.stack([want["y"][7], want["x"][27]])) < tol
    assert r.step([{"id": "x", "tokens": toks["x"][28:29].tolist(), "want": []}], []) is None
    lg = r.step([{"id": "x", "tokens": toks["x"][29:].tolist(), "want": [0]}], ["x"])
    assert Z.rel_err(lg, want["x"][29:]) < tol and not r.slots


def test_limits_are_refused(small):
    for key, value in (("dim", 600), ("kv_rank", 600)):
        bad = copy.deepcopy(Z.SMALL)
        bad["layers"][2]["mixer"][key] = value
        with pytest.raises(ValueError):
            LayeredDecoder.from_config(LayeredConfig(bad), BF16, small.device).engine(max_len=64)
