"""Host logic of the layered decoder designs without a GPU: weight loading, the ragged step with its portions, slots and pages,
the fixed-batch engine, the continuous-batching loop and the trace runner's replay, over CPU stand-ins of the device ops that
are built from the plain implementation (they address pages and state rings the way the kernels do)."""
import json

import pytest
import torch

from oracle import layered_ref as lr
from tests import layers_util as lu


def _rows(rows):
    qo = rows.qo_indptr.tolist()
    for b in range(rows.B):
        yield b, qo[b], qo[b + 1] - qo[b], int(rows.pos0[b])


def embed_pos(tokens, table, pos_table, rows, scale=1.0):
    out = table[tokens].float() * scale
    for _, r, n, pos in _rows(rows):
        if pos_table is not None:
            out[r:r + n] += pos_table[pos:pos + n]
    return out


def resid_norm(x, delta, weight, eps, out_scale=1.0, shift=None, ring=None, rows=None):
    x = x if delta is None else x + delta
    h = lr.rms(x, eps) * weight
    y = h.clone()
    if shift is not None:
        R = ring.shape[1]
        for b, r, n, pos in _rows(rows):
            if n == 0:
                continue
            slot = b if rows.slots is None else int(rows.slots[b])
            before = ring[slot, (pos - 1) % R].clone() if pos else None
            y[r:r + n] = lr.token_shift(h[r:r + n], shift, before)
            for k in range(max(0, n - (R - 1)), n):
                ring[slot, (pos + k) % R] = h[r + k]
    return x, y * out_scale


def extended_attention(qkv, s, k_cache, v_cache, rows, page_indices, page_indptr, max_pages, workspace, **kw):
    out = torch.empty(qkv.shape[0], s.H * s.DV)
    page = k_cache.shape[2]
    for b, r, n, pos in _rows(rows):
        if n == 0:
            continue
        pages = page_indices[int(page_indptr[b]):int(page_indptr[b + 1])].tolist()
        assert len(pages) * page >= pos + n and len(pages) <= max_pages
        q, k, v = qkv[r:r + n].split([s.H * s.D, s.KH * s.D, s.KH * s.DV], 1)
        for j in range(n):
            pg, at = pages[(pos + j) // page], (pos + j) % page
            k_cache[pg, :, at, :s.D] = k[j].view(s.KH, s.D)
            v_cache[pg, :, at, :s.DV] = v[j].view(s.KH, s.DV)
        idx = [(pages[p // page], p % page) for p in range(pos + n)]
        ks = torch.stack([k_cache[pg, :, at, :s.D] for pg, at in idx])
        vs = torch.stack([v_cache[pg, :, at, :s.DV] for pg, at in idx])
        o = lr.attention(q.view(n, s.H, s.D), ks, vs, s.r1, s.r2, s.scale, s.chunk or 1 << 30, s.eps, pos)
        out[r:r + n] = o.flatten(1)
    return out


@pytest.fixture
def layer_ops(monkeypatch):
    from magicdec_amd import harness, ops
    monkeypatch.setattr(ops, "embed_pos", embed_pos)
    monkeypatch.setattr(ops, "resid_norm", resid_norm)
    monkeypatch.setattr(ops, "extended_attention", extended_attention)
    monkeypatch.setattr(ops, "xielu", lambda z, act, out=None: lr.xielu(z, act[0], act[1]))
    monkeypatch.setattr(ops, "argmax", lambda logits: logits.argmax(-1))
    monkeypatch.setattr(ops, "AttnWorkspace", lambda device: None)
    return harness


CFG = lu.config([lu.layer(chunk=20, heads=4, kv_heads=2, dim=12, vdim=20, ff=40), lu.layer(chunk=150, mlp=False, heads=2, kv_heads=1)],
                vocab=90, width=48, max_positions=300, embed_scale=0.8, logit_scale=1.7)


@pytest.fixture(scope="module")
def model(tmp_path_factory):
    return lu.make(tmp_path_factory.mktemp("layers_cpu"), CFG, 3)


def engine(folder, slots, pages=None, max_len=300):
    from magicdec_amd.Engine.SnapKV.backend import LMBackend
    e = LMBackend(dtype=torch.float32, device="cpu")
    e.load_model(folder, use_tp=False)
    e.setup_caches(max_batch_size=slots, max_seq_length=max_len, num_pages=pages)
    for layer, ring in zip(e.model.layers, e.model._rings):
        layer.attention.kv_cache.k_cache.fill_(float("nan"))
        layer.attention.kv_cache.v_cache.fill_(float("nan"))
        ring.fill_(float("nan"))
    return e


@pytest.mark.parametrize("portion_rows", [6, 17, 1000])
def test_ragged_steps_portions_and_reuse(layer_ops, model, monkeypatch, portion_rows):
    from magicdec_amd.Engine import backend_core
    monkeypatch.setattr(backend_core, "PREFILL_ROWS", portion_rows)
    folder, ref = model
    e = engine(folder, slots=3, pages=5)
    for trial in range(2):                              # the second time in slots and pages that were used
        seqs = {k: lu.tokens(n, 90, 10 * trial + n) for k, n in (("a", 140), ("b", 1), ("c", 41))}
        want = {k: ref.logits(v) for k, v in seqs.items()}
        cut = {"a": 133, "b": 1, "c": 22}
        toks, lg = e.step([(k, s[:cut[k]]) for k, s in seqs.items()], [list(range(cut[k])) for k in seqs])
        assert float(lu.row_errors(lg, torch.cat([want[k][:cut[k]] for k in seqs])).max()) < 1e-5
        assert toks.tolist() == [int(want[k][cut[k] - 1].argmax()) for k in seqs]
        e.end("b")
        for t in range(7):
            now = ("c", "a") if t % 2 else ("a", "c")
            _, lg = e.step([(k, seqs[k][cut[k] + t:cut[k] + t + 1]) for k in now], [[0], [0]], sample=False)
            assert float(lu.row_errors(lg, torch.stack([want[k][cut[k] + t] for k in now])).max()) < 1e-5
        e.end("a")
        _, lg = e.step([("c", seqs["c"][29:])], [[0, 11]], sample=False)      # a later portion of a prompt
        assert float(lu.row_errors(lg, want["c"][[29, 40]]).max()) < 1e-5
        e.end("c")
    assert sorted(e.pool.free_pages) == list(range(5)) and sorted(e.pool.free_slots) == [0, 1, 2]


def test_step_refuses_what_it_cannot_run(layer_ops, model):
    e = engine(model[0], slots=2, pages=3)
    for bad in ([("a", [1]), ("a", [2])], [("a", [])], [("a", [90])], [("a", [-1])]):
        with pytest.raises(ValueError):
            e.step(bad)
    with pytest.raises(ValueError, match="position vectors"):
        e.step([("a", [1] * 301)])
    with pytest.raises(RuntimeError, match="step"):
        e.encode(torch.tensor([[1, 2]]))
    with pytest.raises(ValueError, match="position vectors"):
        engine(model[0], slots=1, max_len=301)


def test_fixed_batch_generation(layer_ops, model):
    folder, ref = model
    e = engine(folder, slots=2, max_len=200)
    e.prefill_chunk = 32                                # portions that divide neither the prompt nor the chunks
    prompts = torch.tensor([lu.tokens(101, 90, s) for s in (1, 2)])
    out, steps, _ = layer_ops.run_baseline_batch(e, prompts, 140, -1, -1)
    for b in (0, 1):
        assert out[b, 101:].tolist() == ref.greedy(prompts[b].tolist(), 39)[0]


def test_continuous_batching_order_and_budget(layer_ops, model):
    folder, ref = model
    e = engine(folder, slots=2, pages=3)
    prompts = [lu.tokens(n, 90, n) for n in (120, 3, 130, 40, 1)]
    peak = []
    out, _, _ = layer_ops.run_sequences(e, prompts, 12, on_token=lambda i, t: peak.append(sum(len(s[1]) for s in e.pool.seqs.values())))
    assert max(peak) <= 3 and not e.pool.seqs
    for p, o in zip(prompts, out):
        assert o == ref.greedy(p, 12)[0]


def test_weights_that_do_not_fit_the_config_are_refused(model, tmp_path):
    from magicdec_amd.Engine.SnapKV.backend import LMBackend
    t = lu.tensors(CFG, 1)
    for change, err in ((lambda d: d.pop("l1.shift"), KeyError), (lambda d: d.update(extra=torch.zeros(1)), KeyError),
                        (lambda d: d.update({"l0.mix.o": torch.zeros(48, 81)}), ValueError)):
        d = dict(t)
        change(d)
        folder = lu.write_model(tmp_path / "bad", CFG, d)
        with pytest.raises(err):
            LMBackend(dtype=torch.float32, device="cpu").load_model(folder, use_tp=False)
    with pytest.raises(NotImplementedError, match="tensor parallelism"):
        LMBackend(dtype=torch.float32, device="cpu").load_model(model[0], use_tp=True)


def test_named_configuration_without_a_checkpoint(tmp_path):
    from magicdec_amd.Engine import designs
    spec = designs.find_design(tmp_path / "Furitar-1B" / "model.pth")
    assert spec.dim == 2048 and spec.n_layer == 16
    assert designs.find_design(tmp_path / "Meta-Llama-3.1-8B" / "model.pth") is None
    (tmp_path / "x").mkdir()
    (tmp_path / "x" / "config.json").write_text(json.dumps({"model_type": "llama"}))
    assert designs.find_design(tmp_path / "x" / "model.pth") is None
    (tmp_path / "x" / "config.json").write_text(json.dumps({"architecture": "Nobody"}))
    with pytest.raises(ValueError, match="Nobody"):
        designs.find_design(tmp_path / "x")


def test_replay_resizes_its_pool_for_a_large_batch(layer_ops, model, monkeypatch):
    from magicdec_amd import trace
    monkeypatch.setattr(trace, "MAX_SLOTS", 2)
    folder, ref = model
    r = trace.Replay(folder, torch.float32, 150, device="cpu")
    seqs = [lu.tokens(7, 90, s) for s in range(5)]
    out = r.step({"entries": [{"id": str(k), "tokens": s, "want": [6, 2]} for k, s in enumerate(seqs)],
                  "end": [str(k) for k in range(5)]})
    want = torch.cat([ref.logits(s)[[6, 2]] for s in seqs])
    assert float(lu.row_errors(out, want).max()) < 1e-5
    assert r.step({"entries": [{"id": "z", "tokens": [1], "want": []}], "end": ["z"]}) is None
