"""The latent-attention decoder design on the GPU against the plain implementation (oracle/latent_ref.py): every kernel alone, then
whole models through LMBackend -- prompts, portions, ragged batches, reused pages, long decoding, greedy generation, graphs,
speculative decoding, the trace runner.  Run with -m gpu."""
import json
import os
import subprocess

import pytest
import torch

from oracle import latent_ref as la
from oracle.layered_ref import rms
from tests import latent_util as lu
from tests.conftest import ROOT, parity_report
from tests.test_gpu_layers import dev, feed, greedy_close, i32, ops  # noqa: F401  (fixture and helpers)

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
BF, F32 = torch.bfloat16, torch.float32
TOL = {BF: 0.03, F32: 2e-5}          # row_errors of logits: 16-bit activations / 32-bit throughout


def tol_of(name, dtype):
    """("uneven" has latents of one number: their norm is nearly a sign, which 16-bit rounding moves most)"""
    return TOL[dtype] * (2 if name == "uneven" and dtype == BF else 1)


# ---------------------------------------------------------------------------------------------------------------- kernels
@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("width,mul", [(64, (3, 5)), (100, (2 ** 31 - 1, 2 ** 31 - 19)), (2056, (-7, 11))])
def test_embed_bigram_over_portions(ops, dtype, width, mul):  # noqa: F811
    """Sequences in portions of one, two and many tokens across page borders, in shuffled pages full of other tokens."""
    g = torch.Generator().manual_seed(width)
    V, n_pairs, page, lens = 50, 37, 8, [29, 17, 1]
    E, G = torch.randn(V, width, generator=g).to(dtype), torch.randn(n_pairs + 1, width, generator=g).to(dtype)
    w = (1 + 0.3 * torch.randn(width, generator=g)).to(dtype)
    seqs = [torch.randint(0, V, (n,), generator=g) for n in lens]
    want = [rms(E[s].double() + G[la.bigram_rows(s, None, *mul, n_pairs)].double(), 1e-5) * w.double() for s in seqs]
    for cuts in ([[29], [17], [1]], [[1] * 29, [1] * 17, [1]], [[2, 1, 5, 1, 2, 18], [7, 1, 1, 1, 7], [1]]):
        pages = torch.randperm(16, generator=g).tolist()
        own = [pages[:4], pages[4:7], pages[7:8]]
        history = torch.full((16, page), 13, dtype=torch.int32, device=DEV)
        at = [0, 0, 0]
        for step in range(max(len(c) for c in cuts)):
            live = [b for b in (2, 0, 1) if step < len(cuts[b])]
            n = [cuts[b][step] for b in live]
            qo, ptr, idx = [0], [0], []
            for b, k in zip(live, n):
                qo.append(qo[-1] + k)
                idx += own[b]
                ptr.append(len(idx))
            rows = ops.StepRows(i32(qo), i32([at[b] for b in live]), max(n))
            got = ops.embed_bigram(dev(torch.cat([seqs[b][at[b]:at[b] + k] for b, k in zip(live, n)])), dev(E), dev(G), dev(w), 1e-5, *mul,
                                   history, rows, i32(idx), i32(ptr))
            ref = torch.cat([want[b][at[b]:at[b] + k] for b, k in zip(live, n)])
            assert got.dtype == F32 and torch.allclose(got.cpu().double(), ref, rtol=2e-6, atol=2e-6), (cuts, step)
            for b, k in zip(live, n):
                at[b] += k


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("shape", [(3, 64), (65, 300), (2, 33)])
def test_gelu_mul_and_softcap(ops, dtype, shape):  # noqa: F811
    g = torch.Generator().manual_seed(shape[1])
    z = torch.randn(shape[0], 2 * shape[1], generator=g).mul(4).to(dtype)
    a, b = z[:, :shape[1]], z[:, shape[1]:]
    want = la.gelu_tanh(a.double()) * b.double()
    tol = 2.0 ** -8 if dtype == BF else 1e-5
    zd = dev(z)
    wide = torch.zeros(shape[0], shape[1] + 16, dtype=dtype, device=DEV)
    for out in (None, wide[:, 8:8 + shape[1]]):
        got = ops.gelu_mul(zd[:, :shape[1]], zd[:, shape[1]:], out=out)
        assert torch.allclose(got.cpu().double(), want, rtol=tol, atol=1e-5)
    assert not wide[:, :8].any() and not wide[:, 8 + shape[1]:].any()
    want = la.softcap(z.double(), 2.5)
    assert torch.allclose(ops.softcap_(zd.clone(), 2.5).cpu().double(), want, rtol=tol, atol=1e-5)


@pytest.mark.parametrize("M", [1, 33, 64, 200])
def test_linear_with_gated_gelu_epilogue(ops, M):  # noqa: F811
    """gelu(gate . x) * (up . x) as the epilogue of the three decode GEMMs, into a slice of a wider row."""
    K, ff = 1024, 1024
    g = torch.Generator().manual_seed(M)
    x, w = torch.randn(M, K, generator=g).to(BF), (torch.randn(2 * ff, K, generator=g) * 0.06).to(BF)
    z = x.double() @ w.double().t()
    want = la.gelu_tanh(z[:, :ff]) * z[:, ff:]
    pk, ws = ops.PackedWeight(dev(w), swiglu=True), ops.AttnWorkspace(DEV)
    for name, fn in (("tile", lambda o: ops.fused_linear(dev(x), pk, swiglu=True, gelu=True, out=o)),
                     ("skinny", lambda o: ops.linear(dev(x), pk, swiglu=True, gelu=True, workspace=ws, out=o)),
                     ("block", lambda o: ops.linear_block(dev(x), pk, swiglu=True, gelu=True, workspace=ws, out=o))):
        side = torch.zeros(M, 64 + ff, dtype=BF, device=DEV)
        fn(side[:, 64:])
        assert torch.allclose(side[:, 64:].cpu().double(), want, rtol=2.0 ** -7, atol=5e-3) and not side[:, :64].any(), name
        err = (side[:, 64:].cpu().double() - want).abs() / (want.abs() + 1e-2)
        assert float(err.mean()) < 2e-3, name                       # one rounding of the product, not three


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("M,H,N,K", [(1, 3, 48, 40), (7, 5, 20, 24), (70, 4, 128, 512), (130, 2, 33, 50), (300, 16, 512, 128), (5, 2, 64, 4)])
def test_head_linear(ops, dtype, M, H, N, K):  # noqa: F811
    g = torch.Generator().manual_seed(M)
    x, w = torch.randn(M, H, K + 8, generator=g).to(dtype), (torch.randn(H, N, K, generator=g) * K ** -0.5).to(dtype)
    gate = torch.randn(M, H + 3, generator=g).to(dtype)
    want = torch.stack([x[:, h, :K].double() @ w[h].double().T for h in range(H)], 1)
    tol = dict(rtol=2.0 ** -7, atol=4e-3) if dtype == BF else dict(rtol=1e-5, atol=1e-5)
    out = torch.full((M, H * N + 16), 7.0, dtype=dtype, device=DEV)
    got = ops.head_linear(dev(x)[:, :, :K], dev(w), out[:, 8:8 + H * N].unflatten(1, (H, N)))
    assert torch.allclose(got.cpu().double(), want, **tol) and bool((out[:, :8] == 7).all()) and bool((out[:, 8 + H * N:] == 7).all())
    got = ops.head_linear(dev(x)[:, :, :K], dev(w), torch.empty(M, H, N, dtype=dtype, device=DEV), gate=dev(gate)[:, 3:])
    assert torch.allclose(got.cpu().double(), want * torch.sigmoid(gate[:, 3:].double()).unsqueeze(-1), **tol)


class Seqs:
    """Paged latent rows of several sequences for one layer, pages shuffled and poisoned with NaN."""

    def __init__(self, ops, spec, dtype, lens, page=128, seed=0):  # noqa: F811
        self.ops, self.spec, self.page = ops, spec, page
        npg = [-(-n // page) for n in lens]
        perm = torch.randperm(sum(npg) + 3, generator=torch.Generator().manual_seed(seed)).tolist()
        self.cache = torch.full((len(perm), page, spec.width), float("nan"), dtype=dtype, device=DEV)
        ptr = [0]
        for n in npg:
            ptr.append(ptr[-1] + n)
        self.pages = [perm[ptr[b]:ptr[b + 1]] for b in range(len(lens))]
        self.ws, self.maxp = ops.AttnWorkspace(DEV), max(npg)

    def attend(self, z, q, who, pos, n, gate=None, form="auto"):
        """rows of sequences `who` (n[i] rows from pos[i]) -> (output rows, normalised query latents)"""
        o = self.ops
        qo, idx, ptr = [0], [], [0]
        for b, k in zip(who, n):
            qo.append(qo[-1] + k)
            idx += self.pages[b]
            ptr.append(len(idx))
        rows = o.StepRows(i32(qo), i32(pos), max(n))
        tab = (i32(idx), i32(ptr), self.maxp)
        cq = o.latent_append(dev(z), self.spec, self.cache, rows, *tab)
        ctx = None
        if form == "expanded":
            ctx = o.LatentContext(n, [p + k for p, k in zip(pos, n)], DEV)
            ctx.expanded = lambda s: True
        side = torch.full((qo[-1], self.spec.H * self.spec.vdim + 8), 3.0, dtype=q.dtype, device=DEV)
        out = side[:, :self.spec.H * self.spec.vdim].unflatten(1, (self.spec.H, self.spec.vdim))
        o.latent_attention(dev(q), self.spec, self.cache, rows, *tab, self.ws, out, gate=dev(gate) if gate is not None else None, ctx=ctx,
                           plain=form == "plain")
        assert bool((side[:, self.spec.H * self.spec.vdim:] == 3).all())
        return out.flatten(1).cpu(), cq.cpu()


def attention_case(ops, H, D, RD, VD, Q, R, seed, dtype, lens, score=14.0, yarn=None, dims=None):  # noqa: F811
    """Random rows whose queries ask for chosen places: the unrotated query is the key of that place, scaled to `score`."""
    g = torch.Generator().manual_seed(seed)
    rot = {"dims": RD if dims is None else dims, "base": 500.0}
    if yarn:
        rot["scaling"] = yarn
    tab = ops.RotaryTable(rot["dims"], rot["base"], max(lens) + 5, tuple(yarn[k] for k in ("factor", "original", "fast", "slow")) if yarn else None,
                          device=DEV)
    expand = (torch.randn(H * (D + VD), R, generator=g) * R ** -0.5).to(dtype)
    dqn, kvn = (1 + 0.3 * torch.randn(Q, generator=g)).to(dtype), (1 + 0.3 * torch.randn(R, generator=g)).to(dtype)
    scale, eps = score / D, 1e-5
    spec = ops.LatentSpec(H, D, RD, VD, Q, R, scale, eps, tab, dev(expand), dev(dqn), dev(kvn))
    wk, wv = expand[:H * D].double(), expand[H * D:].double()
    zs, qs, gates, refs, cqs = [], [], [], [], []
    for n in lens:
        z = torch.randn(n, Q + R + RD + H, generator=g).to(dtype)
        c, r = la.latent_keys(z[:, Q:Q + R + RD].double(), kvn.double(), R, rot, eps, 0)
        if dtype == BF:                                              # what the cache holds
            c, r = c.to(BF).double(), r.to(BF).double()
        k = (c @ wk.T).view(n, H, D)
        k = k * (D ** 0.5 / k.norm(dim=-1, keepdim=True))
        q = torch.randn(n, H, D + RD, generator=g).double() * 0.3
        for i in range(n):           # every head asks for one place: near, the first tokens, page and tile borders, far
            targets = [i, max(i - 1, 0), 0, min(1, i), i - i % 128, max(i - i % 128 - 1, 0), i - i % 32, max(i - i % 64 - 1, 0), i // 2, min(i + 1, n - 1)]
            for h in range(H):
                q[i, h, :D] += k[targets[(i + h) % len(targets)], h]
        q = q.flatten(1).to(dtype)
        gate = z[:, Q + R + RD:]
        o = la.latent_attention(q.double(), c, r, wk, wv, H, D, VD, rot, scale, 0)
        zs.append(z)
        qs.append(q)
        gates.append(gate)
        refs.append((o.flatten(1), (o * torch.sigmoid(gate.double()).unsqueeze(-1)).flatten(1)))
        cqs.append(rms(z[:, :Q].double(), eps) * dqn.double())
    return spec, zs, qs, gates, refs, cqs


ATT = [  # H, D, RD, VD, Q, R, yarn, rotated dims
    (4, 32, 16, 40, 48, 64, None, None), (6, 24, 8, 16, 56, 48, lu.YARN, None), (16, 128, 64, 128, 96, 512, None, None),
    (33, 64, 64, 64, 64, 512, lu.YARN, None), (1, 16, 24, 8, 24, 40, lu.YARN, None), (20, 40, 32, 72, 40, 256, None, 16),
    (3, 18, 6, 30, 25, 37, None, None), (5, 100, 20, 90, 64, 130, lu.YARN, None), (8, 128, 64, 192, 64, 400, None, None),
    (2, 192, 64, 256, 32, 200, None, None), (2, 64, 128, 32, 32, 128, None, None), (3, 32, 32, 32, 32, 640, None, None),
    (7, 48, 48, 136, 64, 16, None, None), (2, 256, 16, 264, 40, 96, None, None)]


@pytest.mark.parametrize("H,D,RD,VD,Q,R,yarn,dims", ATT, ids=["-".join(map(str, a[:6])) for a in ATT])
@pytest.mark.parametrize("dtype", [BF, F32])
def test_attention(ops, H, D, RD, VD, Q, R, yarn, dims, dtype):  # noqa: F811
    """Whole prompts in every form; prompts in portions down to single and two tokens; decoding one, two and five rows at a time; a
    second, shorter sequence beside it; with and without gates."""
    lens = [333, 150]
    spec, zs, qs, gates, refs, cqs = attention_case(ops, H, D, RD, VD, Q, R, H * 100 + D, dtype, lens, yarn=yarn, dims=dims)
    tol = 3e-2 if dtype == BF else 3e-5
    worst = {}

    def run(label, s, at, n, who=(0, 1), gated=False, form="auto"):
        who = [b for b in who if n[b] > 0]
        cut = [slice(at[b], at[b] + n[b]) for b in who]
        got, cq = s.attend(torch.cat([zs[b][c] for b, c in zip(who, cut)]), torch.cat([qs[b][c] for b, c in zip(who, cut)]), who,
                           [at[b] for b in who], [n[b] for b in who],
                           torch.cat([gates[b][c] for b, c in zip(who, cut)]) if gated else None, form)
        want = torch.cat([refs[b][gated][c] for b, c in zip(who, cut)])
        err = float((got.double() - want).abs().max()) / max(1.0, float(want.abs().max()))
        worst[label] = max(worst.get(label, 0.0), err)
        assert err <= tol, (label, at, n, err)
        assert torch.allclose(cq.double(), torch.cat([cqs[b][c] for b, c in zip(who, cut)]), rtol=2.0 ** -8 if dtype == BF else 1e-5, atol=1e-5)
    forms = ["auto"] + (["plain"] if dtype == BF else []) + ["expanded"]
    for form in forms:
        run("whole " + form, Seqs(ops, spec, dtype, lens, seed=1), [0, 0], lens, gated=form != "plain", form=form)
    for portion in ((2, 1), (5, 7), (64, 33), (129, 128)):
        s, at, steps = Seqs(ops, spec, dtype, lens, seed=3), [0, 0], 0
        while at[0] < lens[0] or at[1] < lens[1]:
            rest = portion[0] == 2 and steps == 40      # the rest of the two-token portions in one
            n = [lens[b] - at[b] if rest else min(portion[b], lens[b] - at[b]) for b in (0, 1)]
            run("portions", s, at, n, who=(1, 0) if steps % 2 else (0, 1), gated=steps % 3 == 0, form="expanded" if steps % 2 else "auto")
            at = [a + k for a, k in zip(at, n)]
            steps += 1
    for width in (1, 2, 5):
        s = Seqs(ops, spec, dtype, lens, seed=4)
        at = [lens[0] - 6 * width - 30, 125]
        run("prefix", s, [0, 0], at)
        for _ in range(5):
            run("decode", s, at, [width, width])
            at = [a + width for a in at]
    parity_report(f"[latent-attention] H={H} D={D}+{RD} V={VD} R={R} {str(dtype)[6:]} max err " + " ".join(f"{k} {v:.1e}" for k, v in worst.items()))


def test_decoding_across_every_page_and_tile_edge(ops):  # noqa: F811
    """40 tokens decoded one by one from just before a page's end, next to a sequence that starts at its first token."""
    lens = [280, 45]
    for H, D, RD, VD, R in ((4, 32, 16, 40, 64), (16, 64, 64, 64, 512)):
        spec, zs, qs, _, refs, _ = attention_case(ops, H, D, RD, VD, 32, R, 5, BF, lens)
        s = Seqs(ops, spec, BF, lens, seed=9)
        s.attend(zs[0][:236], qs[0][:236], [0], [0], [236])
        for k in range(44):
            at = [236 + k, k]
            got, _ = s.attend(torch.cat([zs[b][at[b]:at[b] + 1] for b in (0, 1)]), torch.cat([qs[b][at[b]:at[b] + 1] for b in (0, 1)]), [0, 1], at, [1, 1])
            want = torch.cat([refs[b][0][at[b]:at[b] + 1] for b in (0, 1)])
            assert float((got.double() - want).abs().max()) < 3e-2 * max(1.0, float(want.abs().max())), (H, k)


def test_long_context_is_split_over_workgroups(ops):  # noqa: F811
    """One sequence: the keys of a decode launch go to many workgroups, whose sums, references and weights are merged; the far key
    that a head asks for lies in another split than the near ones."""
    lens = [2500]
    for H, R, RD in ((8, 512, 64), (40, 128, 32)):
        spec, zs, qs, _, refs, _ = attention_case(ops, H, 64, RD, 64, 32, R, 7, BF, lens, score=18.0)
        s = Seqs(ops, spec, BF, lens, seed=5)
        s.attend(zs[0][:2490], qs[0][:2490], [0], [0], [2490], form="expanded")
        for at in range(2490, 2500):
            got, _ = s.attend(zs[0][at:at + 1], qs[0][at:at + 1], [0], [at], [1])
            assert float((got.double() - refs[0][0][at:at + 1]).abs().max()) < 3e-2 * float(refs[0][0].abs().max()), at


def test_scores_of_any_size(ops):  # noqa: F811
    """Large, tiny and negated scores: the running maximum moves by hundreds, or not at all."""
    for score in (0.01, 90.0, 400.0, -20.0):
        spec, zs, qs, _, refs, _ = attention_case(ops, 4, 64, 16, 64, 32, 96, 11, BF, [200], score=score)
        for form in ("auto", "expanded", "plain"):
            got, _ = Seqs(ops, spec, BF, [200]).attend(zs[0], qs[0], [0], [0], [200], form=form)
            assert torch.isfinite(got.float()).all()
            # 16-bit queries: a score of `score` moves by up to score / 256
            err = (got.double() - refs[0][0]).abs().max(-1).values / float(refs[0][0].abs().max())
            assert float(err.median()) < 0.02 + abs(score) / 400, (score, form, float(err.median()))


def test_rows_beyond_the_page_list_are_dropped_and_counted(ops):  # noqa: F811
    spec, zs, qs, _, _, _ = attention_case(ops, 4, 32, 16, 32, 32, 64, 1, BF, [140])
    s = Seqs(ops, spec, BF, [128])
    guard = s.cache.clone()
    ops.page_overflow_count(reset=True)
    s.attend(zs[0][:126], qs[0][:126], [0], [0], [126])
    s.attend(zs[0][126:131], qs[0][126:131], [0], [126], [5])
    assert ops.page_overflow_count(reset=True) == 3
    others = [p for p in range(s.cache.shape[0]) if p not in s.pages[0]]
    assert torch.equal(s.cache[others].isnan(), guard[others].isnan())


# ----------------------------------------------------------------------------------------------------------------- models
CFG = {
    "small": lu.config([lu.layer(1), lu.layer(2, yarn=lu.YARN, vdim=16), lu.layer(2, yarn=lu.YARN, kv_from=1, vdim=72)]),
    # sizes of one, odd sizes, shared caches of several layers, no feed-forward
    "uneven": lu.config([lu.layer(2, heads=1, dim=7, rot_dim=2, vdim=5, q_rank=9, kv_rank=11, ff=33, yarn=lu.YARN),
                         lu.layer(2, heads=5, dim=40, rot_dim=20, vdim=24, q_rank=30, kv_rank=100, ff=72, yarn=dict(lu.YARN, factor=1.5)),
                         lu.layer(1, heads=3, dim=18, rot_dim=6, vdim=31, q_rank=1, kv_rank=1, mlp=False),
                         lu.layer(2, heads=2, dim=9, rot_dim=20, vdim=33, q_rank=21, kv_rank=100, mlp=False, yarn=dict(lu.YARN, factor=1.5), kv_from=1),
                         lu.layer(2, heads=7, dim=3, rot_dim=2, vdim=8, q_rank=40, kv_rank=11, ff=1, yarn=lu.YARN, kv_from=0)],
                        vocab=211, width=90, eps=1e-3, softcap=5.0, buckets=7, mul_prev=-3, mul_cur=10 ** 9),
    "plain_yarn_less": lu.config([lu.layer(2, heads=6, dim=16, rot_dim=16, vdim=16, q_rank=32, kv_rank=32, ff=64, base=20.0)], vocab=97, width=64,
                                 softcap=100.0, buckets=1, mul_prev=1, mul_cur=1),
    # shapes the hand-written GEMMs take, and prompts that take the expanded form
    "wide": lu.config([lu.layer(1, heads=8, dim=64, rot_dim=32, vdim=64, q_rank=256, kv_rank=480, ff=1024),
                       lu.layer(2, heads=16, dim=48, rot_dim=64, vdim=64, q_rank=384, kv_rank=512, ff=512, yarn=lu.YARN),
                       lu.layer(2, heads=4, dim=128, rot_dim=64, vdim=128, q_rank=128, kv_rank=512, ff=1024, yarn=lu.YARN, kv_from=1)],
                      vocab=512, width=512, buckets=1000),
}
SEED = {k: 20 + i for i, k in enumerate(CFG)}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    root = tmp_path_factory.mktemp("latent")
    return {k: lu.make(root / k, c, SEED[k]) for k, c in CFG.items()}


def serve(folder, dtype, slots=8, pages=None, max_len=1024, **kw):
    from magicdec_amd.Engine.SnapKV.backend import LMBackend
    e = LMBackend(dtype=dtype, device=DEV, **kw)
    e.load_model(folder, use_tp=False)
    e.setup_caches(max_batch_size=slots, max_seq_length=max_len, num_pages=pages)
    return e


def poison(e):
    """NaN into every page: what a sequence reads must be what it wrote itself."""
    for layer in e.model.layers:
        layer.attention.kv_cache.rows.fill_(float("nan"))
    e.model._history.fill_(3)


@pytest.mark.parametrize("name", list(CFG))
@pytest.mark.parametrize("dtype", [F32, BF])
def test_model_prompts_portions_and_decoding(models, name, dtype):
    folder, ref = models[name]
    n = 300
    ids = lu.tokens(n, CFG[name]["vocab"], 77)
    want = ref.logits(ids)
    e = serve(folder, dtype, slots=2, pages=8)
    poison(e)
    worst = {}
    for label, cuts in (("whole", [n]), ("halves", [150, 150]), ("portions", [1, 2, 2, 5, 16, 15, 17, 48, 31, 163]),
                        ("twos", [2] * 40 + [220]), ("decode", [260] + [1] * 40), ("from one token", [1] * 60 + [240])):
        got = feed(e, label, ids, cuts)
        e.end(label)
        worst[label] = float(lu.row_errors(got, want).max())
        assert worst[label] < tol_of(name, dtype), (label, worst[label], lu.row_errors(got, want).argmax())
    parity_report(f"[latent-model] {name} {str(dtype)[6:]} row error " + " ".join(f"{k} {v:.1e}" for k, v in worst.items()))


def test_the_wide_model_takes_the_expanded_form(models, monkeypatch):
    from magicdec_amd import ops as o
    taken = []
    real = o.LatentContext.expanded
    monkeypatch.setattr(o.LatentContext, "expanded", lambda self, s: taken.append(real(self, s)) or taken[-1])
    e = serve(models["wide"][0], BF, slots=1)
    e.step([("a", lu.tokens(300, 512, 1))])
    assert taken == [True, True, True]
    taken.clear()
    e.step([("a", [5])])
    assert taken == [False, False, False]


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("name", ["uneven", "wide"])
def test_residual_after_every_layer(models, name, dtype):
    folder, ref = models[name]
    ids = lu.tokens(90, CFG[name]["vocab"], 5)
    want = []
    ref.step(torch.tensor(ids), ref.new_state(), want)
    e = serve(folder, dtype, slots=1)
    got = []

    def hook(i, x, delta):
        d = delta.sum() if hasattr(delta, "planes") else delta
        got.append((x + d.float()).cpu())
    e.model._layer_hook = hook
    e.step([("a", ids)])
    assert len(got) == len(want)
    for i, (a, b) in enumerate(zip(got, want)):
        assert float(lu.row_errors(a, b).max()) < tol_of(name, dtype), i


@pytest.mark.parametrize("name", ["small", "uneven", "wide"])
@pytest.mark.parametrize("dtype", [F32, BF])
def test_ragged_batches_equal_each_alone(models, name, dtype):
    """Prompts of unequal lengths in one batch, decoded together with sequences that end earlier; then other sequences in the freed
    slots and pages, admitted while some are still decoding."""
    folder, ref = models[name]
    V = CFG[name]["vocab"]
    lens = [1, 2, 127, 128, 129, 30, 257]
    seqs = [lu.tokens(n + 20, V, 100 + n) for n in lens]
    want = [ref.logits(s) for s in seqs]
    e = serve(folder, dtype, slots=7, pages=16)
    poison(e)

    def check(k, lo, got):
        err = lu.row_errors(got.float(), want[k][lo:lo + got.shape[0]])
        assert float(err.max()) < tol_of(name, dtype), (name, k, lo, float(err.max()))
    _, lg = e.step([(k, s[:n]) for k, (s, n) in enumerate(zip(seqs, lens))], [list(range(n)) for n in lens], sample=False)
    at = 0
    for k, n in enumerate(lens):
        check(k, 0, lg[at:at + n])
        at += n
    live = list(range(len(lens)))
    for t in range(20):
        _, lg = e.step([(k, seqs[k][lens[k] + t:lens[k] + t + 1]) for k in live], [[0]] * len(live), sample=False)
        for j, k in enumerate(live):
            check(k, lens[k] + t, lg[j:j + 1])
        if t in (4, 9, 14):
            e.end(live.pop(t % len(live)))
        if t == 15:                                    # two of the sequences once more, in what the others gave back
            again = [k for k in range(len(lens)) if k not in live][:2]
            _, lg = e.step([(f"again{k}", seqs[k]) for k in again], [list(range(len(seqs[k]))) for k in again], sample=False)
            at = 0
            for k in again:
                check(k, 0, lg[at:at + len(seqs[k])])
                at += len(seqs[k])
                e.end(f"again{k}")
    for k in live:
        e.end(k)
    assert len(e.pool.free_pages) == 16 and len(e.pool.free_slots) == 7


def test_long_decoding_crosses_pages(models):
    folder, ref = models["small"]
    ids = lu.tokens(600, 300, 3)
    want = ref.logits(ids)
    e = serve(folder, F32, slots=1)
    got = feed(e, "a", ids, [3] + [1] * 597)
    assert float(lu.row_errors(got, want).max()) < TOL[F32]


def test_far_keys_show(tmp_path):
    """A token asks for one place: the first tokens, page borders, its own neighbourhood, far away -- in prompts and decoded."""
    borders = ((0, 250), (1, 130), (127, 299), (128, 200), (129, 131), (126, 132), (255, 256), (90, 220))
    cfg, t, ids = lu.asking_model(borders=borders)
    folder, ref = lu.write_model(tmp_path / "far", cfg, t), la.LatentRefModel(cfg, t)
    want = ref.logits(ids)
    for dtype in (F32, BF):
        e = serve(folder, dtype, slots=1)
        for label, cuts in (("w", [300]), ("p", [129, 128, 43]), ("d", [120] + [1] * 180)):
            err = lu.row_errors(feed(e, label, ids, cuts), want)
            assert float(err.max()) < (0.05 if dtype == BF else 5e-5), (dtype, label, float(err.max()), int(err.argmax()))
            e.end(label)
    for j, i in borders:                               # a key that is not seen would show
        other = list(ids)
        other[j] = 3
        assert float(lu.row_errors(ref.logits(other), want)[i]) > 0.2


@pytest.mark.parametrize("name", ["small", "uneven", "wide"])
@pytest.mark.parametrize("graphs", [False, True])
def test_greedy_generation_through_the_engine(models, name, graphs):
    """encode + inference of a fixed batch (the baseline loop), eager and with captured decode steps, twice over the same engine;
    decoding crosses pages."""
    from magicdec_amd import harness
    from magicdec_amd.Engine.SnapKV.backend import LMBackend
    folder, ref = models[name]
    V = CFG[name]["vocab"]
    e = LMBackend(dtype=BF, device=DEV)
    e.load_model(folder, use_tp=False)
    if graphs:
        e.compile()
    e.setup_caches(max_batch_size=3, max_seq_length=300)
    for trial in range(2):
        prompts = torch.tensor([lu.tokens(121, V, 50 + trial * 3 + b) for b in range(3)], device=DEV)
        out, steps, _ = harness.run_baseline_batch(e, prompts, 150, -1, -1)
        assert out.shape == (3, 150) and steps == 28
        for b in range(3):
            greedy_close(ref, prompts[b].tolist(), out[b, 121:].tolist())
        if trial == 0:
            first = out
    assert not torch.equal(first, out)
    assert torch.isfinite(e.model.tok_embeddings.weight.float()).all() and e.model.tok_embeddings.weight.stride(0) > 0


@pytest.mark.parametrize("dtype", [F32, BF])
def test_continuous_batching(models, dtype):
    from magicdec_amd import harness
    folder, ref = models["small"]
    prompts = [lu.tokens(n, 300, 900 + n) for n in (5, 130, 1, 64, 260, 33, 128)]
    e = serve(folder, dtype, slots=3, pages=7)
    out, steps, _ = harness.run_sequences(e, prompts, 16, eot=(7,))
    assert not e.pool.seqs and len(e.pool.free_pages) == 7
    for p, o in zip(prompts, out):
        assert len(o) == 16 or o[-1] == 7
        greedy_close(ref, p, o, 0.06 if dtype == BF else 1e-3)


def test_speculative_decoding_with_a_draft_of_the_design(models):
    """The longspec loop with this design as target and as (full-cache) draft; rejected tails need no undo (every state is addressed
    by position), whatever their length."""
    from magicdec_amd import harness
    from magicdec_amd.Engine.SnapKV.backend import LMBackend
    from magicdec_amd.Engine.SnapKV.backend_draft import LMBackend_Draft
    folder, ref = models["wide"]
    prompts = torch.tensor([lu.tokens(121, 512, 40 + b) for b in range(2)], device=DEV)
    for gamma in (3, 18):
        e = LMBackend(dtype=BF, device=DEV, dec_len=gamma + 1)
        e.load_model(folder, use_tp=False)
        e.setup_caches(max_batch_size=2, max_seq_length=256)
        d = LMBackend_Draft(dtype=BF, device=DEV, draft_budget=-1)
        d.load_model(folder, use_tp=False)
        d.setup_caches(max_batch_size=2, max_seq_length=256, draft_budget=-1)
        for forced in (None, lambda st: torch.tensor([2, 1], device=DEV)):
            st, _ = harness.run_longspec_batch(e, d, prompts, gamma, 200, -1, -1, forced_accept_fn=forced)
            if forced is None:
                for b in range(2):
                    greedy_close(ref, prompts[b].tolist(), st.output[b, 121:int(st.num_nodes[b])].tolist())


def test_rolled_back_tokens_leave_no_trace(models):
    """Verify steps of four tokens of which one or two are kept: the logits are those of the kept sequence (pages, and the token
    before in the bigram)."""
    from magicdec_amd.Engine.SnapKV.backend import LMBackend
    folder, ref = models["wide"]
    e = LMBackend(dtype=BF, device=DEV, dec_len=4)
    e.load_model(folder, use_tp=False)
    e.setup_caches(max_batch_size=2, max_seq_length=300)
    seqs = [lu.tokens(170, 512, b) for b in (1, 2)]
    want = [ref.logits(s) for s in seqs]
    e.encode(torch.tensor([s[:120] for s in seqs], device=DEV))
    at = [120, 120]
    for step in range(16):
        keep = [1 + step % 2, 2 - step % 2]
        junk = lu.tokens(8, 512, 1000 + step)
        ids = torch.tensor([seqs[b][at[b]:at[b] + keep[b]] + junk[4 * b + keep[b]:4 * b + 4] for b in (0, 1)], device=DEV)
        e.inference(ids)
        lg = e.model._last_logits.float().view(2, 4, -1)
        for b in (0, 1):
            err = lu.row_errors(lg[b, :keep[b]], want[b][at[b]:at[b] + keep[b]])
            assert float(err.max()) < TOL[BF], (step, b)
            at[b] += keep[b]
        e.cachelens -= i32([4 - k for k in keep])
        e.paged_kv_last_page_len -= i32([4 - k for k in keep])


def test_what_the_design_does_not_have_is_refused(models):
    from magicdec_amd.Engine.SnapKV.backend import LMBackend
    from magicdec_amd.Engine.SnapKV.backend_draft import LMBackend_Draft
    s = LMBackend_Draft(dtype=BF, device=DEV, draft_budget=129)
    s.load_model(models["small"][0], use_tp=False)
    with pytest.raises(NotImplementedError):
        s.setup_caches(max_batch_size=2, max_seq_length=256, draft_budget=129)
    e = LMBackend(dtype=BF, device=DEV)
    e.load_model(models["small"][0], use_tp=False)
    with pytest.raises(NotImplementedError):
        e.setup_caches(max_batch_size=1, max_seq_length=256, kv_dtype="fp8")


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_runner(models, tmp_path, dtype):
    """bin/trace_run as a process: wanted places in any order, several batches, sequences that end early."""
    folder, ref = models["uneven"]
    seqs = {k: lu.tokens(n, 211, n) for k, n in (("a", 140), ("b", 9), ("c", 61))}
    want = {k: ref.logits(v) for k, v in seqs.items()}
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": seqs["a"], "want": [139, 0, 70]}], "end": ["a"]},
             {"step": 1, "entries": [{"id": "b", "tokens": seqs["b"][:5], "want": []},
                                     {"id": "c", "tokens": seqs["c"][:60], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "c", "tokens": seqs["c"][60:], "want": [0]},
                                     {"id": "b", "tokens": seqs["b"][5:6], "want": [0]}], "end": ["c"]}]
    p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", dtype, "--out", str(tmp_path),
                        "--max-tokens", "160"], input="".join(json.dumps(s) + "\n" for s in steps), text=True,
                       capture_output=True, timeout=110)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [ln for ln in p.stdout.splitlines() if ln.startswith("done")] == [f"done {i}" for i in range(3)]
    for s, rows in {0: [("a", 139), ("a", 0), ("a", 70)], 2: [("c", 60), ("b", 5)]}.items():
        got = torch.frombuffer(bytearray((tmp_path / f"{s}.f32").read_bytes()), dtype=F32).view(len(rows), 211)
        ref_rows = torch.stack([want[k][i] for k, i in rows])
        assert float(lu.row_errors(got, ref_rows).max()) < tol_of("uneven", getattr(torch, dtype)) * 1.5, s


def test_command_line_serves_the_design(models, capsys):
    """The baseline command line over a checkpoint folder, fixed batch and ragged."""
    from magicdec_amd import cli
    base = ["--model", models["small"][0], "--rank_group", "0", "--B", "2", "--prefix_len", "100", "--max_len", "128"]
    assert cli.baseline_main(base) > 0
    assert cli.baseline_main(base + ["--ragged", "--dtype", "float32"]) > 0
    assert "sequences :20" in capsys.readouterr().out
