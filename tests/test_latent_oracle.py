"""The plain implementation of the latent-attention decoder's mechanisms (oracle/latent_ref.py): each equation against an
independent evaluation, and -- by planting mistakes in it -- that the inputs of the GPU tests would show them."""
import copy
import math

import pytest
import torch

from oracle import latent_ref as la
from tests import latent_util as lu

F64 = torch.float64


def test_bigram_rows():
    t = torch.tensor([5, 0, 7, 7])
    assert la.bigram_rows(t, None, 131, 17, 50).tolist() == [50, (5 * 131) % 50, (7 * 17) % 50, (7 * 131 + 7 * 17) % 50]
    assert la.bigram_rows(t[1:], 5, 131, 17, 50).tolist() == la.bigram_rows(t, None, 131, 17, 50).tolist()[1:]


def test_rotation_turns_neighbouring_pairs():
    g = torch.Generator().manual_seed(1)
    x = torch.randn(6, 3, 10, generator=g, dtype=F64)
    rot = {"dims": 8, "base": 50.0}
    y = la.rotate(x, rot, 40)
    for t in range(6):
        for i in range(4):
            z = complex(*x[t, 1, 2 * i:2 * i + 2].tolist()) * complex(math.cos((40 + t) * 50.0 ** (-2 * i / 8)), math.sin((40 + t) * 50.0 ** (-2 * i / 8)))
            assert abs(z.real - float(y[t, 1, 2 * i])) < 1e-12 and abs(z.imag - float(y[t, 1, 2 * i + 1])) < 1e-12
    assert torch.equal(y[..., 8:], x[..., 8:])


def test_yarn_frequencies():
    """Slow waves divided by the factor, fast ones untouched, a ramp between; the amplitude grows with the factor."""
    s = {"factor": 4.0, "original": 2048, "fast": 32.0, "slow": 1.0}
    w, amp = la.inverse_freqs({"dims": 64, "base": 10000.0, "scaling": s})
    plain, one = la.inverse_freqs({"dims": 64, "base": 10000.0})
    assert one == 1.0 and abs(amp - (1 + 0.1 * math.log(4))) < 1e-12
    ratio = plain / w
    turns = 2048 * plain / (2 * math.pi)
    assert bool((ratio[turns > 40] - 1 < 1e-12).all()) and bool((ratio[turns < 0.7] > 3.999).all())
    assert bool((ratio[1:] >= ratio[:-1] - 1e-12).all()) and bool(((ratio > 1.01) & (ratio < 3.99)).any())
    # degenerate ramps: everything fast, and everything slow
    w, _ = la.inverse_freqs({"dims": 4, "base": 10.0, "scaling": dict(s, original=10 ** 9)})
    assert torch.allclose(w, la.inverse_freqs({"dims": 4, "base": 10.0})[0])
    w, _ = la.inverse_freqs({"dims": 4, "base": 10.0, "scaling": dict(s, original=0.01)})
    assert float(w[1]) < float(la.inverse_freqs({"dims": 4, "base": 10.0})[0][1]) / 3.9


def test_product_tables_match():
    from magicdec_amd import ops
    for rot in ({"dims": 16, "base": 900.0}, {"dims": 24, "base": 5e5, "scaling": lu.YARN}, {"dims": 2, "base": 10.0, "scaling": lu.YARN}):
        s = rot.get("scaling")
        tab = ops.RotaryTable(rot["dims"], rot["base"], 50, (s["factor"], s["original"], s["fast"], s["slow"]) if s else None, device="cpu")
        x = torch.randn(50, rot["dims"], dtype=F64)
        c, sn = tab.table.double()[..., 0], tab.table.double()[..., 1]
        u, v = x[:, 0::2], x[:, 1::2]
        got = torch.stack([u * c - v * sn, v * c + u * sn], -1).flatten(1)
        assert torch.allclose(got, la.rotate(x, rot, 0), atol=1e-6)


def test_attention_against_scalar_loops():
    g = torch.Generator().manual_seed(3)
    T, H, D, RD, VD, R = 7, 3, 4, 6, 5, 8
    rot = {"dims": RD, "base": 30.0}
    c, r = torch.randn(T, R, generator=g, dtype=F64), torch.randn(T, RD, generator=g, dtype=F64)
    wk, wv = torch.randn(H * D, R, generator=g, dtype=F64), torch.randn(H * VD, R, generator=g, dtype=F64)
    q = torch.randn(4, H * (D + RD), generator=g, dtype=F64)
    out = la.latent_attention(q, c, r, wk, wv, H, D, VD, rot, 0.4, 3)
    qr = la.rotate(q.view(4, H, D + RD)[..., D:], rot, 3)
    for i in range(4):
        for h in range(H):
            w = {}
            for j in range(i + 4):
                k = wk[h * D:(h + 1) * D] @ c[j]
                w[j] = math.exp(0.4 * (float(q.view(4, H, -1)[i, h, :D] @ k) + float(qr[i, h] @ r[j])))
            want = sum(e / sum(w.values()) * (wv[h * VD:(h + 1) * VD] @ c[j]) for j, e in w.items())
            assert torch.allclose(out[i, h], want, atol=1e-10)


def test_activation_and_cap():
    for z in (-6.0, -0.3, 0.0, 1.7, 9.0):
        want = 0.5 * z * (1 + math.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))
        assert abs(float(la.gelu_tanh(torch.tensor(z, dtype=F64))) - want) < 1e-12
    assert abs(float(la.softcap(torch.tensor(40.0, dtype=F64), 30.0)) - 30 * math.tanh(40 / 30)) < 1e-12


CFG = lu.config([lu.layer(1), lu.layer(2, yarn=lu.YARN, vdim=16), lu.layer(1, mlp=False), lu.layer(2, yarn=lu.YARN, kv_from=1, vdim=32, heads=3)],
                vocab=80, width=64)


def test_portions_equal_the_whole_sequence():
    ref = la.LatentRefModel(CFG, lu.tensors(CFG, 1))
    ids = torch.tensor(lu.tokens(29, 80, 2))
    whole = ref.logits(ids)
    for cuts in ([1] * 29, [2] * 14 + [1], [7, 7, 7, 8], [28, 1]):
        st, got, at = ref.new_state(), [], 0
        for n in cuts:
            got.append(ref.step(ids[at:at + n], st))
            at += n
        assert torch.allclose(torch.cat(got), whole, atol=1e-9)


@pytest.mark.parametrize("mistake", ["no_yarn", "no_amplitude", "halves", "position_off", "no_rotation", "no_gate", "own_cache",
                                     "no_bigram_state", "swapped_pair", "no_latent_norm", "gelu_erf", "scaled_yarn_query", "no_cap"])
def test_planted_mistakes_show(mistake, monkeypatch):
    """Every fault the GPU tests are meant to find moves the logits of such a model by far more than rounding."""
    t = lu.tensors(CFG, 4)
    ids = torch.tensor(lu.tokens(60, 80, 5))
    ref = la.LatentRefModel(CFG, t)

    def run(m):
        st = m.new_state()
        return torch.cat([m.step(ids[:33], st), m.step(ids[33:], st)])
    want = run(ref)
    cfg = copy.deepcopy(CFG)
    real_freqs, real_rotate, real_rows = la.inverse_freqs, la.rotate, la.bigram_rows
    limit = 0.03
    if mistake == "no_yarn":
        for L in cfg["layers"]:
            L["mixer"]["rot"].pop("scaling", None)
    elif mistake == "no_amplitude":
        monkeypatch.setattr(la, "inverse_freqs", lambda rot: (real_freqs(rot)[0], 1.0))
    elif mistake == "halves":                                        # first half with second half instead of neighbours
        def halves(x, rot, pos):
            n = rot["dims"]
            perm = torch.stack([torch.arange(n // 2), torch.arange(n // 2) + n // 2], 1).flatten()
            return real_rotate(x[..., perm], rot, pos)
        monkeypatch.setattr(la, "rotate", halves)
    elif mistake == "position_off":                                  # queries one position late
        real = la.latent_attention

        def late(*args):
            monkeypatch.setattr(la, "rotate", lambda x, rot, pos: real_rotate(x, rot, pos + 1))
            try:
                return real(*args)
            finally:
                monkeypatch.setattr(la, "rotate", real_rotate)
        monkeypatch.setattr(la, "latent_attention", late)
    elif mistake == "no_rotation":
        monkeypatch.setattr(la, "rotate", lambda x, rot, pos: x)
    elif mistake == "no_gate":
        monkeypatch.setattr(la.LatentRefModel, "GATED", ())
    elif mistake == "own_cache":                                     # the sharing layer attends to the layer in front of it
        cfg["layers"][3]["mixer"]["kv_from"] = 0
    elif mistake == "no_bigram_state":
        monkeypatch.setattr(la, "bigram_rows", lambda tk, before, a, b, n: real_rows(tk, None, a, b, n))
    elif mistake == "swapped_pair":
        monkeypatch.setattr(la, "bigram_rows", lambda tk, before, a, b, n: real_rows(tk, before, b, a, n))
    elif mistake == "no_latent_norm":
        monkeypatch.setattr(la, "latent_keys", lambda d, w, R, rot, eps, pos: (d[:, :R] * w, real_rotate(d[:, R:], rot, pos)))
    elif mistake == "gelu_erf":
        limit = 3e-4                                                 # (the two forms differ little: the 32-bit run shows it)
        monkeypatch.setattr(la, "gelu_tanh", lambda z: 0.5 * z * (1 + torch.erf(z / math.sqrt(2))))
    elif mistake == "scaled_yarn_query":                             # the amplitude on the whole score
        real = la.latent_attention
        monkeypatch.setattr(la, "latent_attention", lambda q, c, r, wk, wv, h, d, v, rot, s, p: real(
            q, c, r, wk, wv, h, d, v, rot, s * real_freqs(rot)[1] ** 2, p))
    elif mistake == "no_cap":
        monkeypatch.setattr(la, "softcap", lambda z, cap: z)
    got = run(la.LatentRefModel(cfg, t))
    assert float(lu.row_errors(got, want).max()) > limit, mistake


def test_far_keys_stand_out():
    """In the asking model a token's output is that of the one place it asks for: another token there changes it, another token
    beside that place does not."""
    borders = [(0, 250), (127, 299), (128, 200)]
    cfg, t, ids = lu.asking_model(borders=borders)
    ref = la.LatentRefModel(cfg, t)
    want = ref.logits(ids)
    for j, i in borders:
        for at, shows in ((j, True), (j + 4, False), (i - 4, False)):
            other = list(ids)
            other[at] = 3 if other[at] != 3 else 4
            err = float(lu.row_errors(ref.logits(other), want)[i])
            assert (err > 0.2) == shows and (shows or err < 0.02), (j, i, at, err)


def test_config_reader_rejects_what_it_does_not_know():
    from magicdec_amd.Engine.designs import spec_from_config
    spec = spec_from_config(CFG)
    assert spec.layers[3].attention.kv_from == 1 and spec.layers[2].mlp is None and spec.layers[0].attention.gate
    assert not spec.layers[1].attention.gate and spec.layers[1].attention.rotary.yarn.factor == 5.0 and spec.tied_head
    null = copy.deepcopy(CFG)
    null["layers"][0]["mixer"]["kv_from"] = null["layers"][0]["mixer"]["rot"]["scaling"] = None
    assert spec_from_config(null) == spec
    for path, val in ((("extra",), 1), (("layers", 0, "type"), "attention"), (("layers", 0, "mixer", "window"), 3),
                      (("layers", 0, "mlp", "kind"), "routed"), (("layers", 0, "mixer", "heads"), 0), (("architecture",), "Other"),
                      (("norm", "eps"), "x"), (("layers", 0, "mixer", "rot", "dims"), 7), (("layers", 0, "mixer", "rot", "dims"), 10),
                      (("layers", 3, "mixer", "kv_from"), 3), (("layers", 3, "mixer", "kv_from"), 7), (("layers", 3, "mixer", "kv_from"), 0),
                      (("layers", 3, "mixer", "kv_rank"), 40), (("embedding", "bigram", "mul_cur"), 1.5), (("logit_softcap",), 0.0),
                      (("layers", 1, "mixer", "rot", "scaling", "beta"), 1.0)):
        bad = copy.deepcopy(CFG)
        at = bad
        for k in path[:-1]:
            at = at[k]
        at[path[-1]] = val
        with pytest.raises(ValueError):
            spec_from_config(bad)
    chained = copy.deepcopy(CFG)
    chained["layers"].append(copy.deepcopy(chained["layers"][3]))
    chained["layers"][4]["mixer"]["kv_from"] = 3                     # a layer without a cache of its own
    with pytest.raises(ValueError, match="cache of its own"):
        spec_from_config(chained)


def test_which_form_a_step_takes():
    from magicdec_amd import ops

    class Spec:
        H, dim, rot_dim, vdim, kv_rank = 8, 128, 64, 128, 512
        flops = ops.LatentSpec.flops
    s = Spec()
    assert ops.LatentContext([2000, 300], [2000, 300], "cpu").expanded(s)                # prompts
    assert not ops.LatentContext([1, 1], [2000, 300], "cpu").expanded(s)                 # decoding
    assert not ops.LatentContext([100], [50000], "cpu").expanded(s)                      # a short portion far in
    assert ops.LatentContext([1000], [9000], "cpu").expanded(s)
    assert ops.LatentContext([3, 5], [3, 9], "cpu").indptr.tolist() == [0, 3, 12]
    Spec.kv_rank = 32                                                                    # a latent smaller than a head
    assert not ops.LatentContext([2000], [2000], "cpu").expanded(s)
