"""The plain implementation of the layered decoder's mechanisms (oracle/layered_ref.py): each equation against an independent
evaluation, and -- by planting mistakes in it -- that the inputs of the GPU tests would show them."""
import math

import pytest
import torch

from oracle import layered_ref as lr
from tests import layers_util as lu


def test_norm_and_shift():
    x = torch.randn(5, 6, dtype=torch.float64)
    for row, y in zip(x.tolist(), lr.rms(x, 0.5).tolist()):
        r = math.sqrt(sum(v * v for v in row) / 6 + 0.5)
        assert max(abs(a / r - b) for a, b in zip(row, y)) < 1e-12
    mu = torch.rand(6, dtype=torch.float64)
    y = lr.token_shift(x, mu)
    assert torch.allclose(y[0], x[0] * (1 - mu)) and torch.allclose(y[3], x[3] + (x[2] - x[3]) * mu)
    parts = torch.cat([lr.token_shift(x[:2], mu), lr.token_shift(x[2:], mu, x[1])])
    assert torch.allclose(parts, y)


def test_xielu_matches_the_scalar_formula():
    p, q = 0.4, -0.7
    for z in (-30.0, -2.0, -1e-3, -1e-9, 0.0, 1e-6, 0.3, 5.0):
        sp = lambda v: math.log1p(math.exp(v))             # noqa: E731
        want = sp(p) * z * z + z / 2 if z > 0 else (0.5 + sp(q)) * (math.expm1(z) - z) + z / 2
        got = float(lr.xielu(torch.tensor([z], dtype=torch.float64), torch.tensor(p), torch.tensor(q)))
        assert abs(got - want) < 1e-6 * max(1, abs(want))


def test_attention_against_scalar_loops():
    g = torch.Generator().manual_seed(3)
    T, H, G, D, VD, chunk, scale, eps = 11, 4, 2, 6, 5, 4, 0.7, 1e-5
    q, k, v = (torch.randn(T, n, d, generator=g, dtype=torch.float64) for n, d in ((H, D), (G, D), (G, VD)))
    r1, r2 = torch.rand(H, generator=g, dtype=torch.float64), torch.rand(H, generator=g, dtype=torch.float64)
    out = lr.attention(q, k, v, r1, r2, scale, chunk, eps)
    for i in range(T):
        for h in range(H):
            e = {}
            for j in range(T):
                if j > i or i // chunk != j // chunk:
                    continue
                qn = q[i, h] / math.sqrt(float((q[i, h] ** 2).mean()) + eps)
                kn = k[j, h // 2] / math.sqrt(float((k[j, h // 2] ** 2).mean()) + eps)
                e[j] = math.exp(float(qn @ kn) * scale - float(r1[h]) * math.log(1 + float(r2[h]) * (i - j)))
            den = 1 + sum(e.values())
            want = sum(w / den * v[j, h // 2] for j, w in e.items())
            assert torch.allclose(out[i, h], want, atol=1e-10)


def test_portions_equal_the_whole_sequence():
    cfg = lu.config([lu.layer(chunk=7), lu.layer(mlp=False, chunk=5)], vocab=50, width=24, max_positions=40)
    ref = lr.RefModel(cfg, lu.tensors(cfg, 1))
    ids = torch.tensor(lu.tokens(29, 50, 2))
    whole = ref.logits(ids)
    for cuts in ([1] * 29, [2] * 14 + [1], [7, 7, 7, 8], [28, 1]):
        st, got, at = ref.new_state(), [], 0
        for n in cuts:
            got.append(ref.step(ids[at:at + n], st))
            at += n
        assert torch.allclose(torch.cat(got), whole, atol=1e-9)


@pytest.mark.parametrize("mistake", ["chunk_minus", "chunk_plus", "no_sink", "no_bias", "bias_off_by_one", "no_qk_norm",
                                     "no_shift_state", "wrong_group"])
def test_planted_mistakes_show(mistake, monkeypatch):
    """Every fault the GPU tests are meant to find moves the logits of such a model by far more than their tolerance (2 % in
    16 bits)."""
    cfg = lu.config([lu.layer(chunk=16, scale=0.35, heads=4, kv_heads=2) for _ in range(2)], vocab=80, width=64, max_positions=64)
    t = lu.tensors(cfg, 4)
    for i in range(2):
        t[f"l{i}.mix.r1"] *= 2
        t[f"l{i}.mix.r2"] *= 4
    ids = torch.tensor(lu.tokens(50, 80, 5))
    ref = lr.RefModel(cfg, t)
    st = ref.new_state()
    want = torch.cat([ref.step(ids[:33], st), ref.step(ids[33:], st)])
    real, real_softmax = lr.attention, lr.sink_softmax
    if mistake in ("chunk_minus", "chunk_plus"):
        by = -1 if mistake == "chunk_minus" else 1
        monkeypatch.setattr(lr, "attention", lambda q, k, v, r1, r2, s, c, e, p=0: real(q, k, v, r1, r2, s, c + by, e, p))
    elif mistake == "no_sink":
        monkeypatch.setattr(lr, "sink_softmax", lambda s: torch.softmax(s, -1))
    elif mistake == "no_bias":
        monkeypatch.setattr(lr, "distance_bias", lambda r1, r2, d: 0 * d)
    elif mistake == "bias_off_by_one":
        monkeypatch.setattr(lr, "distance_bias", lambda r1, r2, d: r1 * torch.log(1 + r2 * (d + 1)))
    elif mistake == "no_qk_norm":
        def plain(q, k, v, r1, r2, s, c, e, p=0):
            monkeypatch.setattr(lr, "rms", lambda x, eps: x)
            try:
                return real(q, k, v, r1, r2, s, c, e, p)
            finally:
                monkeypatch.setattr(lr, "rms", rms)
        rms = lr.rms
        monkeypatch.setattr(lr, "attention", plain)
    elif mistake == "no_shift_state":
        shift = lr.token_shift
        monkeypatch.setattr(lr, "token_shift", lambda h, mu, before=None: shift(h, mu, None))
    elif mistake == "wrong_group":
        monkeypatch.setattr(lr, "attention",
                            lambda q, k, v, r1, r2, s, c, e, p=0: real(q, k.flip(1), v.flip(1), r1, r2, s, c, e, p))
    st = ref.new_state()
    got = torch.cat([ref.step(ids[:33], st), ref.step(ids[33:], st)])
    assert float(lu.row_errors(got, want).max()) > 0.06, mistake
    assert real_softmax is not None


def test_config_reader_rejects_what_it_does_not_know():
    from magicdec_amd.Engine.designs import spec_from_config
    cfg = lu.config([lu.layer(), lu.layer(mlp=False, heads=3, kv_heads=1, dim=20, vdim=12)])
    spec = spec_from_config(cfg)
    assert spec.layers[1].mlp is None and spec.layers[1].attention.heads == 3 and spec.layers[0].attention.chunk == 48
    for path, val in ((("extra",), 1), (("layers", 0, "type"), "other"), (("layers", 0, "mixer", "window"), 3),
                      (("layers", 0, "mlp", "kind"), "gated"), (("layers", 0, "mixer", "heads"), 3),
                      (("architecture",), "Other"), (("width",), 0), (("norm", "eps"), "x")):
        bad = lu.config([lu.layer(), lu.layer()])
        at = bad
        for k in path[:-1]:
            at = at[k]
        at[path[-1]] = val
        with pytest.raises(ValueError):
            spec_from_config(bad)
    missing = lu.config([lu.layer()])
    del missing["logit_scale"]
    with pytest.raises(ValueError, match="logit_scale"):
        spec_from_config(missing)


def test_sequence_pool_hands_slots_and_pages_out_again():
    from magicdec_amd.Engine.backend_core import SequencePool
    pool = SequencePool(2, 5, 128)
    pool.grow("a", 130)
    pool.grow("b", 1)
    a, b = pool.seqs["a"], pool.seqs["b"]
    assert len(a[1]) == 2 and len(b[1]) == 1 and len(set(a[1] + b[1])) == 3 and a[0] != b[0]
    pool.grow("b", 127)
    assert len(b[1]) == 1 and pool.length("b") == 128
    pool.grow("b", 1)
    assert len(b[1]) == 2 and not pool.fits(1)             # no slot left
    with pytest.raises(RuntimeError, match="slot"):
        pool.grow("c", 1)
    with pytest.raises(RuntimeError, match="pages"):
        pool.grow("b", 300)
    old = list(a[1])
    pool.release("a")
    pool.grow("c", 129)
    assert pool.seqs["c"][1] == old and pool.seqs["c"][0] == 0 and pool.length("a") == 0
