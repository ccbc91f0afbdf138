"""Host logic of the latent-attention decoder design without a GPU: weight loading, shared caches, the ragged step with its portions
and pages, the fixed-batch engine, the continuous-batching loop, over CPU stand-ins of the device ops that are built from the plain
implementation (they address pages the way the kernels do)."""
import pytest
import torch

from oracle import latent_ref as la
from oracle.layered_ref import rms
from tests import latent_util as lu
from tests.test_layers_cpu import _rows, resid_norm


def _pages(page_indices, page_indptr, b):
    return page_indices[int(page_indptr[b]):int(page_indptr[b + 1])].tolist()


def embed_bigram(tokens, table, pairs, norm_weight, eps, mul_before, mul_token, history, rows, page_indices, page_indptr):
    out = torch.empty(tokens.numel(), table.shape[1])
    page = history.shape[1]
    for b, r, n, pos in _rows(rows):
        pg = _pages(page_indices, page_indptr, b)
        before = int(history[pg[(pos - 1) // page], (pos - 1) % page]) if pos else None
        tk = tokens[r:r + n]
        out[r:r + n] = rms(table[tk] + pairs[la.bigram_rows(tk, before, mul_before, mul_token, pairs.shape[0] - 1)], eps) * norm_weight
        for j in range(n):
            history[pg[(pos + j) // page], (pos + j) % page] = int(tk[j])
    return out


class RotaryTable:
    def __init__(self, dims, base, max_pos, scaling=None, device=None):
        self.rot = {"dims": dims, "base": base}
        if scaling is not None:
            self.rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
        self.max_pos, self.pairs = max_pos, dims // 2


def latent_append(z, s, cache, rows, page_indices, page_indptr, max_pages):
    if s.kv_norm is not None:
        for b, r, n, pos in _rows(rows):
            pg = _pages(page_indices, page_indptr, b)
            assert len(pg) * cache.shape[1] >= pos + n and len(pg) <= max_pages
            c, k = la.latent_keys(z[r:r + n, s.q_rank:s.q_rank + s.kv_rank + s.rot_dim], s.kv_norm, s.kv_rank, s.rotary.rot, s.eps, pos)
            for j in range(n):
                cache[pg[(pos + j) // cache.shape[1]], (pos + j) % cache.shape[1], :s.kv_rank + s.rot_dim] = torch.cat([c[j], k[j]])
    return rms(z[:, :s.q_rank], s.eps) * s.dq_norm


def latent_attention(q, s, cache, rows, page_indices, page_indptr, max_pages, workspace, out, gate=None, ctx=None):
    for b, r, n, pos in _rows(rows):
        if n == 0:
            continue
        pg = _pages(page_indices, page_indptr, b)
        held = torch.cat([cache[p] for p in pg])[:pos + n]
        o = la.latent_attention(q[r:r + n], held[:, :s.kv_rank], held[:, s.kv_rank:s.kv_rank + s.rot_dim], s.expand[:s.H * s.dim],
                                s.expand[s.H * s.dim:], s.H, s.dim, s.vdim, s.rotary.rot, s.scale, pos)
        out[r:r + n] = o * torch.sigmoid(gate[r:r + n]).unsqueeze(-1) if gate is not None else o
    if ctx is not None:
        assert ctx.new == [n for _, _, n, _ in _rows(rows)] and ctx.ctx == [pos + n for _, _, n, pos in _rows(rows)]
    return out


@pytest.fixture
def latent_ops(monkeypatch):
    from magicdec_amd import harness, ops
    for name, fn in (("embed_bigram", embed_bigram), ("resid_norm", resid_norm), ("RotaryTable", RotaryTable), ("latent_append", latent_append),
                     ("latent_attention", latent_attention), ("latent_row_width", lambda r, d: r + d + 3),
                     ("softcap_", la.softcap), ("argmax", lambda logits: logits.argmax(-1)), ("AttnWorkspace", lambda device: None),
                     ("gelu_mul", lambda a, b, out: out.copy_(la.gelu_tanh(a) * b))):
        monkeypatch.setattr(ops, name, fn)
    return harness


CFG = lu.config([lu.layer(2, heads=2, dim=10, rot_dim=6, vdim=12, q_rank=20, kv_rank=16, ff=40, yarn=lu.YARN), lu.layer(1, heads=3, mlp=False),
                 lu.layer(2, heads=5, dim=6, rot_dim=6, vdim=20, q_rank=14, kv_rank=16, ff=30, yarn=lu.YARN, kv_from=0)], vocab=90, width=48)


@pytest.fixture(scope="module")
def model(tmp_path_factory):
    return lu.make(tmp_path_factory.mktemp("latent_cpu"), CFG, 3)


def engine(folder, slots, pages=None, max_len=300):
    from magicdec_amd.Engine.SnapKV.backend import LMBackend
    e = LMBackend(dtype=torch.float32, device="cpu")
    e.load_model(folder, use_tp=False)
    e.setup_caches(max_batch_size=slots, max_seq_length=max_len, num_pages=pages)
    for layer in e.model.layers:
        layer.attention.kv_cache.rows.fill_(float("nan"))
    e.model._history.fill_(17)
    return e


def test_layers_share_one_cache_and_the_head_is_the_embedding(latent_ops, model):
    e = engine(model[0], slots=2)
    a, b, c = (layer.attention for layer in e.model.layers)
    assert c.kv_cache is a.kv_cache and b.kv_cache is not a.kv_cache and c.kv_norm is None and c.cuts == [14, 0, 0]
    assert e.model.output.weight is e.model.tok_embeddings.weight and e.model._rowmajor_in_decode(e.model.output.weight)
    assert e.model._xspec[0].rotary is e.model._xspec[2].rotary and e.model.rollback_depth() is None


@pytest.mark.parametrize("portion_rows", [6, 17, 1000])
def test_ragged_steps_portions_and_reuse(latent_ops, model, monkeypatch, portion_rows):
    from magicdec_amd.Engine import backend_core
    monkeypatch.setattr(backend_core, "PREFILL_ROWS", portion_rows)
    folder, ref = model
    e = engine(folder, slots=3, pages=5)
    e.model.prefill_rows = portion_rows
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


def test_fixed_batch_generation(latent_ops, model):
    folder, ref = model
    e = engine(folder, slots=2, max_len=200)
    e.prefill_chunk = 32
    prompts = torch.tensor([lu.tokens(101, 90, s) for s in (1, 2)])
    out, steps, _ = latent_ops.run_baseline_batch(e, prompts, 140, -1, -1)
    for b in (0, 1):
        assert out[b, 101:].tolist() == ref.greedy(prompts[b].tolist(), 39)[0]


def test_continuous_batching(latent_ops, model):
    folder, ref = model
    e = engine(folder, slots=2, pages=3)
    prompts = [lu.tokens(n, 90, n) for n in (120, 3, 130, 1)]
    out, _, _ = latent_ops.run_sequences(e, prompts, 9)
    for p, o in zip(prompts, out):
        assert o == ref.greedy(p, 9)[0]


def test_weights_that_do_not_fit_the_config_are_refused(model, tmp_path):
    from magicdec_amd.Engine.SnapKV.backend import LMBackend
    t = lu.tensors(CFG, 1)
    for change, err in ((lambda d: d.pop("l1.mix.g"), KeyError), (lambda d: d.update({"l2.mix.dkv": d["l0.mix.dkv"].clone()}), KeyError),
                        (lambda d: d.update({"l0.mix.uk": d["l0.mix.uk"][:-1]}), ValueError), (lambda d: d.update(head=d["embed"].clone()), KeyError)):
        d = dict(t)
        change(d)
        folder = lu.write_model(tmp_path / "bad", CFG, d)
        with pytest.raises(err):
            LMBackend(dtype=torch.float32, device="cpu").load_model(folder, use_tp=False)
    with pytest.raises(NotImplementedError, match="tensor parallelism"):
        LMBackend(dtype=torch.float32, device="cpu").load_model(model[0], use_tp=True)


def test_named_configurations(tmp_path):
    from magicdec_amd.Engine import designs
    spec = designs.find_design(tmp_path / "Bufodra-8B" / "model.pth")
    assert spec.design == "Bufodra" and spec.dim == 4096 and spec.layers[3].attention.kv_from == 1
    assert [s.attention.kv_from for s in spec.layers[:8]] == [None, None, None, 1, None, None, None, 5]
