"""Zapipel without a GPU: configuration, registry, weights, index tables, and the oracle itself."""
import copy
import os

import pytest
import torch

import _zapipel as Z
import zapipel_oracle as oracle
from eventgpt_amd.models import LayeredConfig, LayeredDecoder
from eventgpt_amd.models.registry import load_model, resolve
from eventgpt_amd.runtime import mixers
from eventgpt_amd.runtime.mixers import RowBatch, Sequence_


def test_config_reads_every_size():
    c = LayeredConfig(Z.MIXED)
    assert (c.vocab_size, c.hidden_size, c.norm_eps, c.logit_scale, c.logit_softcap, c.embedding_scale) == (83, 100, 3e-4, 0.7, 4.0, 1.0)
    assert c.design.norm == "layer" and c.design.post_norm and all(l.post_norm for l in c.layers)
    m = c.layers[1].mixer
    assert (m.heads, m.dim, m.vdim, m.kv_rank, m.q_rank, m.scale, m.kv_from) == (18, 33, 16, 100, 70, 0.12, None)
    assert [l.mixer.kv_from for l in c.layers] == [None, None, 0, 1, None, 0]
    e = c.layers[4].mlp
    assert (e.experts, e.top, e.ff, e.act) == (9, 1, 8, "silu") and c.layers[2].mlp is None and c.layers[1].mlp.ff == 72
    s = c.parameter_shapes()
    assert s["l0.mix.dkv"] == (40, 100) and s["l0.mix.dkv.norm"] == (40,) and "l2.mix.dkv" not in s and "l2.mix.dkv.norm" not in s
    assert s["l1.mix.uk"] == (18 * 33, 100) and s["l1.mix.uv"] == (18 * 16, 100) and s["l1.mix.g"] == (18, 100)
    assert s["l1.mix.uq"] == (18 * 33, 70) and s["l1.mix.o"] == (100, 18 * 16)
    assert s["l4.mlp.router"] == (9, 100) and s["l4.mlp.router.b"] == (9,) and s["l4.mlp.e8.down"] == (100, 8)
    assert s["l0.norm1b"] == (100,) and "l2.norm2" not in s and "l2.norm2b" not in s and s["l3.norm2b"] == (100,)


@pytest.mark.parametrize("path,value", [
    (("layers", 1, "mixer", "rope"), 4),
    (("layers", 1, "mixer", "kv_from"), 1),            # itself
    (("layers", 1, "mixer", "kv_from"), 0),            # latents of another size
    (("layers", 5, "mixer", "kv_from"), 2),            # a layer without latents of its own
    (("layers", 0, "mixer", "kv_from"), 3),            # a later layer
    (("layers", 0, "mlp", "kind"), "sparse"),
    (("layers", 0, "mlp", "router", "top"), 6),
    (("layers", 0, "mlp", "expert", "bias"), True),
    (("layers", 0, "type"), "mamba2"),                 # another design's
    (("logit_softcap",), -1.0),
    (("width",), 0),
])
def test_config_refuses_what_it_does_not_know(path, value):
    d = copy.deepcopy(Z.MIXED)
    at = d
    for k in path[:-1]:
        at = at[k]
    at[path[-1]] = value
    with pytest.raises(ValueError):
        LayeredConfig(d)
    d = copy.deepcopy(Z.MIXED)
    del d["logit_scale"]
    with pytest.raises(ValueError):
        LayeredConfig(d)


def test_registry_and_save_load_round_trip(tmp_path):
    assert resolve({"architecture": "Zapipel"}).model is LayeredDecoder and resolve({"architecture": "Zapipel"}).modality == "text"
    m = Z.build(dtype=torch.bfloat16)
    m.save_pretrained(str(tmp_path))
    for dtype in (torch.bfloat16, torch.float32):
        r = load_model(str(tmp_path), dtype, "cpu")
        assert isinstance(r, LayeredDecoder) and r.tensors.keys() == m.tensors.keys()
        assert all(torch.equal(r.tensors[n].float(), t.float()) for n, t in m.tensors.items())
    bad = copy.deepcopy(Z.MIXED)
    bad["layers"][0]["mlp"]["router"]["experts"] = 4
    LayeredConfig(bad).save_pretrained(str(tmp_path))
    with pytest.raises(ValueError):                    # a router with one expert more
        load_model(str(tmp_path), torch.bfloat16, "cpu")


def test_latent_padding():
    assert [mixers.pad_latent(n) for n in (1, 64, 65, 128, 129, 512)] == [64, 64, 128, 128, 256, 512]


def test_causal_tables():
    """Every query row is in one run and one work item; the buffer holds all keys of its sequence, in order."""
    seqs, row = [], 0
    for slot, (start, n) in enumerate([(0, 1), (0, 150), (3, 2), (99, 210), (7, 64)]):
        seqs.append(Sequence_(slot, row, n, start))
        row += n
    runs, items, copies, kv_rows = RowBatch("cpu", False, seqs=seqs).causal_tables()
    where = {}
    for slot, first, dst, n in copies.tolist():
        assert first == 0 and n == seqs[slot].start + seqs[slot].rows
        where.update({dst + i: (slot, i) for i in range(n)})
    assert sorted(where) == list(range(kv_rows))
    owner = {s.row0 + r: (s.slot, s.start + r) for s in seqs for r in range(s.rows)}
    for table in ([r[:4] for r in runs], items.tolist()):
        seen = set()
        for q0, n, k0, off in table:
            for i in range(n):
                slot, p = owner[q0 + i]
                assert q0 + i not in seen and where[k0] == (slot, 0) and p == off + i and where[k0 + p] == (slot, p)
                seen.add(q0 + i)
        assert seen == set(owner)
    assert all(n <= 64 for _, n, _, _ in items.tolist())


def test_latents_are_gathered_once_and_one_sequence_needs_no_copy():
    cache = torch.arange(3 * 9 * 4.).view(3, 9, 4)
    calls = []

    def gather(c, copies, rows):
        calls.append(rows)
        return torch.cat([c[s, a:a + n] for s, a, _, n in copies.tolist()])
    two = RowBatch("cpu", False, seqs=[Sequence_(2, 0, 3, 4), Sequence_(0, 3, 2, 0)])
    want = torch.cat([cache[2, :7], cache[0, :2]])
    assert torch.equal(two.latents(cache, gather), want) and two.latents(cache, gather) is two.latents(cache, gather) and calls == [9]
    one = RowBatch("cpu", False, seqs=[Sequence_(1, 0, 3, 4)]).latents(cache, gather)
    assert torch.equal(one, cache[1, :7]) and one.data_ptr() == cache[1].data_ptr() and calls == [9]


def test_when_a_portion_attends_over_the_cache():
    class M:
        R, D = 512, 128
    absorbs = mixers.LatentAttentionMixer.absorbs

    def pack(*seqs):
        return RowBatch("cpu", False, seqs=[Sequence_(i, 0, n, start) for i, (start, n) in enumerate(seqs)])
    assert absorbs(M, pack((5000, 2))) and absorbs(M, pack((5000, 16), (70, 2)))
    assert not absorbs(M, pack((5000, 600))) and not absorbs(M, pack((0, 2))) and not absorbs(M, pack((5000, 2), (0, 600)))


def test_oracle_far_keys_sharing_and_experts():
    """The oracle shows what it must: an early token reaches a late one, a shared latent is the owner's, an expert that is
    not chosen does not matter, and the logits are causal and capped."""
    m = Z.build()
    t = Z.prompt(30, 83, 0)
    w = Z.weights(m)
    a = oracle.forward(m.config.raw, w, t)
    assert torch.allclose(a[:17], oracle.forward(m.config.raw, w, t[:17]), rtol=0, atol=1e-12) and float(a.abs().max()) < 4.0
    u = t.clone()
    u[0] = (u[0] + 1) % 83
    assert not torch.equal(a[29], oracle.forward(m.config.raw, w, u)[29])
    q, k, v = (torch.randn(9, 2, 4, generator=torch.Generator().manual_seed(s), dtype=torch.float64) for s in range(3))
    o = oracle.causal_attention(q, k, v, 0.5)
    s = torch.nn.functional.scaled_dot_product_attention(q.transpose(0, 1), k.transpose(0, 1), v.transpose(0, 1), is_causal=True, scale=0.5)
    assert torch.allclose(o, s.transpose(0, 1))
    which, f = oracle.route(torch.tensor([[1.0, 3.0, 2.0, 3.0]], dtype=torch.float64), 3)
    assert which.tolist() == [[1, 3, 2]] and torch.allclose(f, torch.softmax(torch.tensor([[3.0, 3.0, 2.0]], dtype=torch.float64), -1))
    x = torch.randn(4, 6, dtype=torch.float64) + 5
    n = oracle.layer_norm(x, 1e-3, torch.ones(6))
    assert torch.allclose(n, torch.nn.functional.layer_norm(x, (6,), eps=1e-3))


def test_engine_needs_a_gpu():
    if torch.cuda.is_available():
        pytest.skip("a GPU is present")
    from eventgpt_amd import build
    if not os.path.exists(build.LAYERED_SO_PATH):
        pytest.skip("extension not built")
    with pytest.raises(RuntimeError):
        Z.build().engine()
