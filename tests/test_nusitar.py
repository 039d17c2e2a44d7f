"""Layered decoders without a GPU: configuration, registry, weights, index tables, and the oracle itself."""
import copy
import json
import os

import pytest
import torch

import _nusitar as N
import nusitar_oracle as oracle
from eventgpt_amd.models import EventChatConfig, EventChatModel, LayeredConfig, LayeredDecoder
from eventgpt_amd.models.registry import load_model, read_config, resolve
from eventgpt_amd.runtime import mixers
from eventgpt_amd.runtime.mixers import RowBatch, Sequence_


def test_config_reads_every_size():
    c = LayeredConfig(N.MIXED)
    assert (c.vocab_size, c.hidden_size, c.norm_eps, c.embedding_scale) == (83, 100, 3e-5, 1.7)
    assert [l.type for l in c.layers] == ["mamba2", "parallel", "parallel", "mamba2", "parallel", "mamba2"]
    left = c.layers[1].mixer.left
    assert (left.heads, left.kv_heads, left.dim, left.vdim, left.scale, left.rot_dims, left.rot_base, left.chunk) == \
        (6, 2, 20, 28, 0.31, 12, 700.0, 13)
    assert c.layers[2].mlp is None and c.layers[3].mlp.ff == 52
    s = c.parameter_shapes()
    assert s["l0.mix.in"] == (2 * 120 + 2 * 3 * 24 + 6, 100) and s["l0.mix.conv"] == (120 + 144, 3)
    assert s["l1.mix.left.o"] == (100, 6 * 28) and s["l1.mix.right.g"] == (72, 100) and s["l1.mix.left.q.norm"] == (120,)
    assert "l0.norm2" not in s and "l1.norm2" in s and "l2.mlp.gate" not in s


@pytest.mark.parametrize("path,value", [
    (("layers", 1, "mixer", "left", "bias"), True),
    (("layers", 1, "mixer", "left", "kv_heads"), 4),
    (("layers", 1, "mixer", "left", "rot", "dims"), 22),
    (("layers", 1, "mlp", "kind"), "moe"),
    (("layers", 0, "mixer", "norm_groups"), 7),
    (("layers", 0, "type"), "mamba3"),
    (("width",), 0),
])
def test_config_refuses_what_it_does_not_know(path, value):
    d = copy.deepcopy(N.MIXED)
    at = d
    for k in path[:-1]:
        at = at[k]
    at[path[-1]] = value
    with pytest.raises(ValueError):
        LayeredConfig(d)


def test_registry_picks_the_class(tmp_path):
    assert resolve({"architecture": "Nusitar"}).model is LayeredDecoder
    assert resolve({"model_type": "EventChat_llama"}).model is EventChatModel
    with pytest.raises(ValueError):
        resolve({"model_type": "something else"})
    EventChatConfig.tiny().save_pretrained(str(tmp_path))
    entry, cfg = read_config(str(tmp_path))
    assert entry.modality == "event" and isinstance(cfg, EventChatConfig)


def test_save_load_round_trip(tmp_path):
    m = N.build(dtype=torch.bfloat16)
    m.save_pretrained(str(tmp_path))
    for dtype in (torch.bfloat16, torch.float32):
        r = load_model(str(tmp_path), dtype, "cpu")
        assert isinstance(r, LayeredDecoder) and r.tensors.keys() == m.tensors.keys()
        assert all(torch.equal(r.tensors[n].float(), t.float()) for n, t in m.tensors.items())
    # a checkpoint of other shapes is refused, also where only the first dimension differs
    bad = json.loads(json.dumps(N.MIXED))
    bad["layers"][0]["mixer"]["conv"] = 4
    LayeredConfig(bad).save_pretrained(str(tmp_path))
    with pytest.raises(ValueError):
        load_model(str(tmp_path), torch.bfloat16, "cpu")
    bad = json.loads(json.dumps(N.MIXED))
    bad["vocab"] += 1
    LayeredConfig(bad).save_pretrained(str(tmp_path))
    with pytest.raises(ValueError):
        load_model(str(tmp_path), torch.bfloat16, "cpu")


def test_engine_needs_a_gpu():
    if torch.cuda.is_available():
        pytest.skip("a GPU is present")
    from eventgpt_amd import build
    if not os.path.exists(build.LAYERED_SO_PATH):
        pytest.skip("extension not built")
    with pytest.raises(RuntimeError):
        N.build().engine()


def test_padding_helpers():
    w = torch.arange(12.).view(6, 2)
    p = mixers.pad_rows(w, 2, 3, 4)
    assert p.shape == (8, 2) and torch.equal(p[:3], w[:3]) and torch.equal(p[4:7], w[3:]) and p[3].abs().sum() == 0
    c = mixers.pad_cols(w.t().contiguous(), 2, 3, 4)
    assert torch.equal(c, p.t())
    assert [mixers.pad_value(n) for n in (1, 32, 33, 64, 65)] == [32, 32, 64, 64, 128]
    assert [mixers.pad_attn_head(n) for n in (1, 64, 65, 128, 129)] == [64, 64, 128, 128, 192]


@pytest.mark.parametrize("size", [1, 2, 5, 7, 64, 100, 1000])
def test_chunk_tables_cover_every_query_once(size):
    """Every query row is in one run and one work item, and its visible keys in the key buffer are the ones a chunk
    mask allows: the buffer rows [chunk key row, chunk key row + position in the chunk] hold its chunk's positions."""
    seqs, row = [], 0
    for slot, (start, n) in enumerate([(0, 1), (0, 150), (3, 2), (99, 210), (7, 64)]):
        seqs.append(Sequence_(slot, row, n, start))
        row += n
    rb = RowBatch("cpu", False, seqs=seqs)
    runs, items, row_kv, keep, copies, kv_rows = rb.chunk_tables(size)
    where = {}                                     # key buffer row -> (slot, position)
    if copies is not None:
        for slot, first, dst, n in copies.tolist():
            start = seqs[slot].start
            for i in range(n):
                where[dst + i] = (slot, start // size * size + first + i)
    for s in seqs:
        for r in range(s.rows):
            assert int(row_kv[s.row0 + r]) not in where
            where[int(row_kv[s.row0 + r])] = (s.slot, s.start + r)
            p, end = s.start + r, s.start + s.rows
            assert bool(keep[s.row0 + r]) == (p // size == end // size)
    assert sorted(where) == list(range(kv_rows))
    owner = {s.row0 + r: (s.slot, s.start + r) for s in seqs for r in range(s.rows)}
    for table in ([(q + i * n, n, k + i * n, off) for q, n, k, off, reps in runs for i in range(reps)], items.tolist()):
        seen = set()
        for q0, n, k0, off in table:
            for i in range(n):
                slot, p = owner[q0 + i]
                assert q0 + i not in seen and p % size == off + i
                seen.add(q0 + i)
                assert [where[k0 + j] for j in range(off + i + 1)] == \
                    [(slot, j) for j in range(p // size * size, p + 1)]
        assert seen == set(owner)
    assert all(n <= 64 for _, n, _, _ in items.tolist())


@pytest.mark.parametrize("L", [64, 128])
def test_scan_tables(L):
    seqs = [Sequence_(3, 0, 130, 0), Sequence_(1, 130, 2, 50), Sequence_(0, 132, 64, 0)]
    rb = RowBatch("cpu", False, seqs=seqs + [Sequence_(2, 196, 3, 7), Sequence_(4, 199, 1, 0)], scan_chunk=L)
    assert rb.tails.tolist() == [[0, 130, 3, 0], [130, 2, 1, 50], [132, 64, 0, 0], [196, 3, 2, 7], [199, 1, 4, 0]]
    assert rb.pos.tolist()[126:134] == [126, 127, 128, 129, 50, 51, 0, 1]
    # flags: first chunk from the zero state / last chunk of the sequence, and the parities of start and end
    at = 0
    for (c0, n, slot, flags), s in zip(rb.scan_seqs.tolist(), rb.seqs):
        assert (c0, n, slot) == (at, -(-s.rows // L), s.slot)
        assert flags == int(s.start == 0) + 2 * (s.start % 2) + 4 * ((s.start + s.rows) % 2)
        for c in range(n):
            assert rb.chunks.tolist()[at + c] == [s.row0 + c * L, min(L, s.rows - c * L), s.slot,
                                                  int(c == n - 1) + 2 * ((s.start + s.rows) % 2)]
        at += n
    assert at == rb.chunks.shape[0]


def test_oracle_chunk_mask_and_state():
    """The oracle shows what it must: a token in an earlier chunk moves the matrix memory but not the attention."""
    g = torch.Generator().manual_seed(0)
    q, k, v = (torch.randn(9, 2, 4, generator=g, dtype=torch.float64) for _ in range(3))
    a = oracle.chunked_attention(q, k, v, 0.5, 4)
    k2 = k.clone()
    k2[3] += 1
    b = oracle.chunked_attention(q, k2, v, 0.5, 4)
    assert torch.equal(a[:3], b[:3]) and not torch.equal(a[3], b[3]) and torch.equal(a[4:], b[4:])
    i, f = torch.randn(9, 2, generator=g, dtype=torch.float64), -torch.rand(9, 2, generator=g, dtype=torch.float64)
    x, y = oracle.mlstm_scan(q, k, v, i, f), oracle.mlstm_scan(q, k2, v, i, f)
    assert torch.equal(x[:3], y[:3]) and not torch.equal(x[8], y[8])


def test_oracle_logits_are_causal():
    m = N.build()
    t = N.prompt(40, 83, 0)
    a = N.oracle_logits(m, t)
    b = N.oracle_logits(m, t[:25])
    assert torch.allclose(a[:25], b, rtol=0, atol=1e-12)


def test_text_cli_checks_its_prompt(tmp_path):
    from eventgpt_amd.cli.inference import run
    N.build(dtype=torch.bfloat16).save_pretrained(str(tmp_path))
    for extra in (["--token_ids", "1,83"], [], ["--token_ids", "1", "--use_4bit"]):
        with pytest.raises(SystemExit):
            run(["--model_path", str(tmp_path), "--device", "cpu"] + extra)
    with pytest.raises(SystemExit):
        run(["--random_init", "tiny", "--query", "x"])
