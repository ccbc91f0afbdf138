"""The layered decoder designs on the GPU against the plain implementation (oracle/layered_ref.py): every kernel alone, then
whole models through LMBackend -- prompts, portions, ragged batches, reused slots and pages, long decoding, greedy generation,
graphs, speculative decoding, the trace runner.  Run with -m gpu."""
import json
import os
import subprocess
import sys

import pytest
import torch

from oracle import layered_ref as lr
from tests import layers_util as lu
from tests.conftest import ROOT, parity_report

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
BF, F32, F64 = torch.bfloat16, torch.float32, torch.float64
TOL = {BF: 0.025, F32: 2e-5}         # row_errors of logits: 16-bit activations / 32-bit throughout


@pytest.fixture(scope="module")
def ops():
    from magicdec_amd import ops as _ops
    _ops._lib.load()
    return _ops


def dev(t, dtype=None):
    return (t if dtype is None else t.to(dtype)).to(DEV)


def i32(v):
    return torch.tensor(v, dtype=torch.int32, device=DEV)


# ---------------------------------------------------------------------------------------------------------------- kernels
@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("width", [64, 100, 2056])
def test_embed_pos(ops, dtype, width):
    g = torch.Generator().manual_seed(width)
    E, P = torch.randn(50, width, generator=g).to(dtype), torch.randn(40, width, generator=g).to(dtype)
    n, pos = [3, 1, 7], [0, 39, 5]
    ids = torch.randint(0, 50, (11,), generator=g)
    rows = ops.StepRows(i32([0, 3, 4, 11]), i32(pos), 7)
    at = [p + j for p, k in zip(pos, n) for j in range(k)]
    want = E[ids].float() * 1.7 + P[at].float()
    got = ops.embed_pos(dev(ids), dev(E), dev(P), rows, 1.7).cpu()
    assert got.dtype == F32 and torch.allclose(got, want, rtol=1e-6, atol=1e-6)
    assert torch.equal(ops.embed_pos(dev(ids), dev(E), None, rows).cpu(), E[ids].float())


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("width,planes", [(64, 0), (100, 0), (768, 3), (2048, 8), (4096, 1), (5120, 5), (1100, 0), (2056, 2)])
def test_resid_norm(ops, dtype, width, planes):
    g = torch.Generator().manual_seed(width + planes)
    M = 37
    x = torch.randn(M, width, generator=g) * 3
    w = (1 + 0.3 * torch.randn(width, generator=g)).to(dtype)
    if planes:
        pl = torch.randn(planes, M, width, generator=g)
        delta, dsum = ops.Planes(dev(pl)), pl.double().sum(0)
    else:
        d = torch.randn(M, width, generator=g).to(dtype)
        delta, dsum = dev(d), d.double()
    xo, y = ops.resid_norm(dev(x), delta, dev(w), 1e-3, out_scale=0.5)
    want_x = x.double() + dsum
    want_y = lr.rms(want_x, 1e-3) * w.double() * 0.5
    assert xo.dtype == F32 and y.dtype == dtype
    assert torch.allclose(xo.cpu().double(), want_x, rtol=1e-6, atol=2e-6)
    tol = 2.0 ** -8 if dtype == BF else 2e-6
    assert torch.allclose(y.cpu().double(), want_y, rtol=tol, atol=tol * 1e-2 if dtype == BF else 2e-6)
    same, y2 = ops.resid_norm(xo, None, dev(w), 1e-3, out_scale=0.5)
    assert same is xo and torch.equal(y2, y)                                    # no delta: the same row, the same norm


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("width,ring", [(64, 4), (100, 16), (2048, 16)])
def test_token_shift_over_portions(ops, dtype, width, ring):
    """Three sequences in portions of 1, 2, ring - 1, ring, ring + 1 and many rows, slots not in batch order: every row equals
    the whole sequence's, bit for bit when it is cut otherwise."""
    g = torch.Generator().manual_seed(width)
    lens, slots = [61, 40, 3], [2, 0, 1]
    w, mu = (1 + 0.3 * torch.randn(width, generator=g)).to(dtype), torch.rand(width, generator=g).to(dtype)
    xs = [torch.randn(n, width, generator=g) for n in lens]
    ds = [torch.randn(n, width, generator=g).to(dtype) for n in lens]

    def run(cuts_of):
        state = torch.full((3, ring, width), float("nan"), device=DEV)
        got = [[] for _ in lens]
        at = [0] * 3
        for step in range(max(len(c) for c in cuts_of)):
            live = [b for b in range(3) if step < len(cuts_of[b])]
            n = [cuts_of[b][step] for b in live]
            qo = [0]
            for v in n:
                qo.append(qo[-1] + v)
            rows = ops.StepRows(i32(qo), i32([at[b] for b in live]), max(n), i32([slots[b] for b in live]))
            x = torch.cat([xs[b][at[b]:at[b] + k] for b, k in zip(live, n)])
            d = torch.cat([ds[b][at[b]:at[b] + k] for b, k in zip(live, n)])
            before = state.clone()
            _, y = ops.resid_norm(dev(x), dev(d), dev(w), 1e-5, shift=dev(mu), ring=state, rows=rows)
            if max(n) < ring:                    # a repeated step reads what the first one read
                again = state.clone()
                _, y2 = ops.resid_norm(dev(x), dev(d), dev(w), 1e-5, shift=dev(mu), ring=again, rows=rows)
                assert torch.equal(y2, y) and torch.equal(again.nan_to_num(7), state.nan_to_num(7))
            del before
            for j, b in enumerate(live):
                got[b].append(y[qo[j]:qo[j + 1]].cpu())
                at[b] += n[j]
        return [torch.cat(v) for v in got]
    whole = run([[n] for n in lens])
    for b, n in enumerate(lens):
        h = lr.rms(xs[b].double() + ds[b].double(), 1e-5) * w.double()
        want = lr.token_shift(h, mu.double())
        tol = 2.0 ** -8 if dtype == BF else 3e-6
        assert torch.allclose(whole[b].double(), want, rtol=tol, atol=tol)
    for cuts in ([[1] * 61, [1] * 40, [1] * 3], [[2] * 30 + [1], [2] * 20, [2, 1]],
                 [[ring - 1, 1, ring, 61 - 2 * ring], [ring + 1, 39 - ring], [3]]):
        for a, b in zip(run(cuts), whole):
            assert torch.equal(a, b)


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("shape", [(5, 64), (33, 100), (300, 1024)])
def test_xielu(ops, dtype, shape):
    z = torch.randn(*shape, generator=torch.Generator().manual_seed(1)) * 3
    z[0, :8] = torch.tensor([0.0, -0.0, 1e-4, -1e-4, -1e-7, 20.0, -20.0, -90.0])
    z, act = z.to(dtype), torch.tensor([0.4, -0.9])
    want = lr.xielu(z.double(), act[0].double(), act[1].double())
    got = ops.xielu(dev(z), dev(act))
    tol = 2.0 ** -8 if dtype == BF else 1e-6
    assert bool(((got.cpu().double() - want).abs() <= tol * want.abs() + 1e-6).all())
    zz = dev(z)
    assert torch.equal(ops.xielu(zz, dev(act), out=zz), got)


@pytest.mark.parametrize("M", [1, 33, 64, 200])
def test_linear_with_xielu_epilogue_and_planes(ops, M):
    """The activation as an epilogue of the three decode GEMMs, and their products left as fp32 planes."""
    K, N = 1024, 2048
    g = torch.Generator().manual_seed(M)
    x, w = torch.randn(M, K, generator=g).to(BF), (torch.randn(N, K, generator=g) * 0.05).to(BF)
    act = torch.tensor([-0.3, 0.8])
    z = x.double() @ w.double().t()
    want = lr.xielu(z, act[0].double(), act[1].double())
    pk, ws = ops.PackedWeight(dev(w)), ops.AttnWorkspace(DEV)
    for name, y in (("tile", ops.fused_linear(dev(x), pk, xielu=dev(act))),
                    ("skinny", ops.linear(dev(x), pk, workspace=ws, xielu=dev(act))),
                    ("block", ops.linear_block(dev(x), pk, workspace=ws, xielu=dev(act)))):
        assert torch.allclose(y.cpu().double(), want, rtol=2.0 ** -7, atol=2e-3), name
    for kind in ops.PLANES_KINDS:
        n = ops.linear_planes_count(kind, M, N, K)
        assert n > 0
        p = ops.linear_planes(dev(x), pk, kind, ws)
        assert p.n == n and torch.allclose(p.sum().cpu().double(), z, rtol=1e-5, atol=1e-4), kind
    assert ops.linear_planes_count("tile", 64, 100, 128) == 0 and ops.linear_planes_count("block", 300, 2048, 1024) == 0


class Seqs:
    """Paged K/V of several sequences for one attention layer, pages shuffled and poisoned with NaN."""

    def __init__(self, ops, spec, dtype, lens, page=128, seed=0):
        self.ops, self.spec, self.page, self.dtype = ops, spec, page, dtype
        npg = [-(-n // page) for n in lens]
        perm = torch.randperm(sum(npg) + 3, generator=torch.Generator().manual_seed(seed)).tolist()
        self.kc = torch.full((len(perm), spec.KH, page, ops.head_pad(spec.D)), float("nan"), dtype=dtype, device=DEV)
        self.vc = torch.full((len(perm), spec.KH, page, ops.head_pad(spec.DV)), float("nan"), dtype=dtype, device=DEV)
        ptr = [0]
        for n in npg:
            ptr.append(ptr[-1] + n)
        self.pages, self.indptr = [perm[ptr[b]:ptr[b + 1]] for b in range(len(lens))], ptr
        self.ws = ops.AttnWorkspace(DEV)
        self.maxp = max(npg)

    def attend(self, qkv, who, pos, n, fuse=True, plain=False):
        """qkv rows of sequences `who` (n[i] rows from pos[i]) -> output rows"""
        qo, idx, ptr = [0], [], [0]
        for b, k in zip(who, n):
            qo.append(qo[-1] + k)
            idx += self.pages[b]
            ptr.append(len(idx))
        rows = self.ops.StepRows(i32(qo), i32(pos), max(n))
        return self.ops.extended_attention(dev(qkv), self.spec, self.kc, self.vc, rows, i32(idx), i32(ptr), self.maxp, self.ws,
                                           fuse=fuse, plain=plain).cpu()


def attention_case(ops, H, KH, D, DV, chunk, seed, dtype, lens, score=12.0, r=(0.9, 0.4)):
    """Random rows whose matched query / key pairs stand out (their score is `score`, the others are ~ score / sqrt(D))."""
    g = torch.Generator().manual_seed(seed)
    r1 = r[0] * (0.5 + torch.rand(H, generator=g))
    r2 = r[1] * (0.5 + torch.rand(H, generator=g))
    scale = score / D
    spec = ops.XattnSpec(H, KH, D, DV, scale, 1e-5, chunk, True, True, dev(r1), dev(r2), 1.02 * score)
    seqs = []
    for n in lens:
        q, k, v = (torch.randn(n, h, d, generator=g) for h, d in ((H, D), (KH, D), (KH, DV)))
        for i in range(n):           # every query of head h asks for one key: near, at its chunk's edges, just outside, far
            lo = i // chunk * chunk if chunk else 0
            targets = [i, max(i - 1, 0), lo, max(lo - 1, 0), lo + (i - lo) // 2, 0, i - i % 128, max(i - i % 128 - 1, 0)]
            for h in range(H):
                j = targets[(i + h) % len(targets)]
                q[i, h] = k[j, h // (H // KH)] + 0.05 * q[i, h]
        seqs.append(tuple(t.to(dtype) for t in (q, k, v)))
    ref = [lr.attention(q.double(), k.double(), v.double(), r1.double(), r2.double(), scale, chunk or 1 << 30, 1e-5)
           for q, k, v in seqs]
    rows = [torch.cat([t.flatten(1) for t in s], 1) for s in seqs]
    return spec, rows, [t.flatten(1) for t in ref]


ATT = [  # H, KH, D, DV, chunk
    (4, 2, 32, 32, 48), (10, 2, 88, 56, 190), (8, 2, 64, 64, 130), (5, 5, 40, 24, 33), (7, 1, 20, 36, 1), (16, 1, 64, 128, 257),
    (12, 4, 80, 112, 300), (4, 4, 128, 128, 129), (24, 1, 128, 64, 511), (3, 1, 192, 160, 77), (2, 2, 256, 256, 100),
    (33, 1, 32, 64, 64), (2, 1, 300, 40, 90), (2, 1, 50, 270, 90), (4, 2, 64, 64, 0)]


@pytest.mark.parametrize("H,KH,D,DV,chunk", ATT, ids=["-".join(map(str, a)) for a in ATT])
@pytest.mark.parametrize("dtype", [BF, F32])
def test_attention(ops, H, KH, D, DV, chunk, dtype):
    """Whole prompts; prompts in portions; decoding one, two and five rows at a time (with and without the append inside the
    attention launch); a second, shorter sequence beside it."""
    lens = [389, 170]
    spec, rows, ref = attention_case(ops, H, KH, D, DV, chunk, H * 1000 + D, dtype, lens)
    tol = 1.5e-2 if dtype == BF else 2e-5

    def check(name, got, want):
        err = float((got.double() - want).abs().max())
        assert err <= tol * max(1.0, float(want.abs().max())), (name, err)
        return err
    s = Seqs(ops, spec, dtype, lens, seed=1)
    errs = [check("whole", s.attend(torch.cat(rows), [0, 1], [0, 0], lens), torch.cat(ref))]
    if dtype == BF:
        s = Seqs(ops, spec, dtype, lens, seed=2)
        errs.append(check("plain", s.attend(torch.cat(rows), [0, 1], [0, 0], lens, plain=True), torch.cat(ref)))
    for portion in ((2, 1), (5, 7), (64, 33), (129, 128)):
        s = Seqs(ops, spec, dtype, lens, seed=3)
        at = [0, 0]
        n_steps = 0
        while at[0] < lens[0] or at[1] < lens[1]:
            if portion[0] == 2 and n_steps == 60:       # the rest of the two-token portions in one
                n = [lens[b] - at[b] for b in (0, 1)]
            else:
                n = [min(portion[b], lens[b] - at[b]) for b in (0, 1)]
            who = [b for b in (0, 1) if n[b] > 0]
            got = s.attend(torch.cat([rows[b][at[b]:at[b] + n[b]] for b in who]), who, [at[b] for b in who], [n[b] for b in who])
            check(("portion", portion, tuple(at)), got, torch.cat([ref[b][at[b]:at[b] + n[b]] for b in who]))
            for b in who:
                at[b] += n[b]
            n_steps += 1
    for width in (1, 2, 5):
        for fuse in (True, False):
            s = Seqs(ops, spec, dtype, lens, seed=4)
            start = [lens[0] - 6 * width - 20, lens[1] - 6 * width - 20]
            s.attend(torch.cat([rows[b][:start[b]] for b in (0, 1)]), [0, 1], [0, 0], start)
            for k in range(6):
                at = [start[b] + k * width for b in (1, 0)]
                got = s.attend(torch.cat([rows[b][a:a + width] for b, a in zip((1, 0), at)]), [1, 0], at, [width, width], fuse=fuse)
                errs.append(check(("decode", width, fuse, k), got, torch.cat([ref[b][a:a + width] for b, a in zip((1, 0), at)])))
    parity_report(f"[layers-attention] H={H} KH={KH} D={D} DV={DV} chunk={chunk} {str(dtype)[6:]} max err {max(errs):.2e}")


def test_attention_across_every_chunk_and_page_edge(ops):
    """Decode 40 tokens across chunk borders that fall on, just before and just behind page and tile borders; every query asks
    for the last key of the previous chunk or the first of its own."""
    for chunk in (31, 32, 33, 127, 128, 129):
        lens = [150, 290]
        spec, rows, ref = attention_case(ops, 4, 2, 64, 64, chunk, chunk, BF, lens)
        s = Seqs(ops, spec, BF, lens, seed=chunk)
        start = [110, 250]
        s.attend(torch.cat([rows[b][:start[b]] for b in (0, 1)]), [0, 1], [0, 0], start)
        for k in range(40):
            at = [v + k for v in start]
            got = s.attend(torch.cat([rows[b][at[b]:at[b] + 1] for b in (0, 1)]), [0, 1], at, [1, 1])
            want = torch.cat([ref[b][at[b]:at[b] + 1] for b in (0, 1)])
            assert float((got.double() - want).abs().max()) < 1.5e-2 * max(1.0, float(want.abs().max())), (chunk, k)


def test_attention_splits_agree(ops):
    """One sequence, a long chunk: the decode launch splits the keys over workgroups."""
    lens = [1500]
    spec, rows, ref = attention_case(ops, 4, 1, 64, 64, 1490, 3, BF, lens)
    s = Seqs(ops, spec, BF, lens, seed=5)
    s.attend(rows[0][:1480], [0], [0], [1480])
    for at in range(1480, 1500):
        got = s.attend(rows[0][at:at + 1], [0], [at], [1])
        assert float((got.double() - ref[0][at:at + 1]).abs().max()) < 1.5e-2 * float(ref[0].abs().max()), at


def test_sink_takes_the_weight_of_low_scores(ops):
    """Queries opposite to every key: the sink holds nearly all the weight, the output is nearly 0 (and not the mean of v)."""
    g = torch.Generator().manual_seed(0)
    H, D, n = 2, 64, 40
    k = torch.randn(1, D, generator=g).expand(n, D) + 0.01 * torch.randn(n, D, generator=g)
    v = 1 + torch.rand(n, D, generator=g)
    qkv = torch.cat([-k, -k, k, v], 1)
    r = dev(torch.zeros(H))
    for dtype in (BF, F32):
        spec = ops.XattnSpec(H, 1, D, D, 8.0 / D, 1e-5, 0, True, True, r, r, 8.2)
        rows = qkv.to(dtype)
        out = Seqs(ops, spec, dtype, [n]).attend(rows, [0], [0], [n])
        t = rows.double()
        ref = lr.attention(t[:, :H * D].view(n, H, D), t[:, H * D:H * D + D].view(n, 1, D), t[:, -D:].view(n, 1, D),
                           torch.zeros(H), torch.zeros(H), 8.0 / D, 1 << 30, 1e-5).flatten(1)
        assert float(ref.abs().max()) < 0.05 and torch.allclose(out.double(), ref, rtol=2e-2, atol=1e-4)


def test_attention_with_a_score_bound_of_any_size(ops):
    """Large scores: the matrix-core kernels move their reference (bound 60..100), beyond it the plain kernel takes over; a
    negative bias coefficient raises the bound; an unknown bound is the plain kernel."""
    for score, bound in ((20.0, 20.4), (75.0, 76.5), (95.0, 97.0), (150.0, 153.0), (20.0, 0.0)):
        spec, rows, ref = attention_case(ops, 4, 2, 64, 32, 40, 9, BF, [100], score=score)
        spec.score_bound = bound
        got = Seqs(ops, spec, BF, [100]).attend(rows[0], [0], [0], [100])
        # q and k are rounded to 16 bits after their norm: a score of `score` moves by up to score / 256
        assert float((got.double() - ref[0]).abs().max()) < (0.02 + score / 400) * float(ref[0].abs().max()), score
        assert torch.isfinite(got.float()).all()


def test_rows_beyond_the_page_list_are_dropped_and_counted(ops):
    spec, rows, _ = attention_case(ops, 4, 2, 64, 64, 300, 1, BF, [140])
    for fuse in (True, False):
        s = Seqs(ops, spec, BF, [128])
        guard = s.kc.clone()
        ops.page_overflow_count(reset=True)
        s.attend(rows[0][:126], [0], [0], [126])
        s.attend(rows[0][126:131], [0], [126], [5], fuse=fuse)
        assert ops.page_overflow_count(reset=True) == 3
        others = [p for p in range(s.kc.shape[0]) if p not in s.pages[0]]
        assert torch.equal(s.kc[others].isnan(), guard[others].isnan())


# ----------------------------------------------------------------------------------------------------------------- models
CFG = {
    "small": lu.config([lu.layer(chunk=48), lu.layer(chunk=48), lu.layer(chunk=48)], embed_scale=0.7, logit_scale=1.6),
    "uneven": lu.config([lu.layer(heads=5, kv_heads=1, dim=40, vdim=24, ff=200, chunk=37),
                         lu.layer(heads=4, kv_heads=4, dim=64, vdim=96, mlp=False, chunk=150),
                         lu.layer(heads=6, kv_heads=3, dim=20, vdim=36, ff=72, chunk=1),
                         lu.layer(heads=2, kv_heads=1, dim=96, vdim=64, ff=320, chunk=1000, scale=0.21)],
                        vocab=211, width=168, eps=1e-3, embed_scale=1.3, logit_scale=0.4, max_positions=700),
    "odd": lu.config([lu.layer(heads=3, kv_heads=3, dim=18, vdim=30, ff=75, chunk=65), lu.layer(heads=3, kv_heads=1, dim=34, vdim=10, ff=31)],
                     vocab=97, width=90, max_positions=400),
    # shapes the hand-written GEMMs take: fused epilogues, K-split planes, the append inside the attention
    "wide": lu.config([lu.layer(heads=8, kv_heads=2, dim=64, vdim=64, ff=1024, chunk=200),
                       lu.layer(heads=16, kv_heads=2, dim=32, vdim=64, ff=512, chunk=96)], vocab=512, width=512),
}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    root = tmp_path_factory.mktemp("layers")
    return {k: lu.make(root / k, c, 10 + i) for i, (k, c) in enumerate(CFG.items())}


def engine(folder, dtype, slots=8, pages=None, max_len=None, cfg=None, **kw):
    from magicdec_amd.Engine.SnapKV.backend import LMBackend
    e = LMBackend(dtype=dtype, device=DEV, **kw)
    e.load_model(folder, use_tp=False)
    limit = e.model.spec.max_positions
    e.setup_caches(max_batch_size=slots, max_seq_length=min(limit, max_len or limit), num_pages=pages)
    return e


def poison(e):
    """NaN into every page and ring: what a sequence reads must be what it wrote itself."""
    for layer, ring in zip(e.model.layers, e.model._rings):
        layer.attention.kv_cache.k_cache.fill_(float("nan"))
        layer.attention.kv_cache.v_cache.fill_(float("nan"))
        ring.fill_(float("nan"))


def feed(e, sid, ids, cuts, want=True):
    out, at = [], 0
    for n in cuts:
        _, lg = e.step([(sid, ids[at:at + n])], [list(range(n))], sample=False)
        out.append(lg.float())
        at += n
    assert at == len(ids)
    return torch.cat(out)


@pytest.mark.parametrize("name", list(CFG))
@pytest.mark.parametrize("dtype", [F32, BF])
def test_model_prompts_portions_and_decoding(models, name, dtype):
    folder, ref = models[name]
    n = 300
    ids = lu.tokens(n, CFG[name]["vocab"], 77)
    want = ref.logits(ids)
    e = engine(folder, dtype, slots=2, pages=8)
    poison(e)
    worst = {}
    for label, cuts in (("whole", [n]), ("halves", [150, 150]), ("portions", [1, 2, 2, 5, 16, 15, 17, 48, 31, 163]),
                        ("twos", [2] * 40 + [220]), ("decode", [260] + [1] * 40), ("from one token", [1] * 60 + [240])):
        got = feed(e, label, ids, cuts)
        e.end(label)
        worst[label] = float(lu.row_errors(got, want).max())
        assert worst[label] < TOL[dtype], (label, worst[label], lu.row_errors(got, want).argmax())
    parity_report(f"[layers-model] {name} {str(dtype)[6:]} row error " + " ".join(f"{k} {v:.1e}" for k, v in worst.items()))


@pytest.mark.parametrize("dtype", [F32, BF])
def test_residual_after_every_layer(models, dtype):
    folder, ref = models["uneven"]
    ids = lu.tokens(90, 211, 5)
    want = []
    ref.step(torch.tensor(ids), ref.new_state(), want)
    e = engine(folder, dtype, slots=1)
    got = []

    def hook(i, x, delta):
        d = delta.sum() if hasattr(delta, "planes") else delta
        got.append((x + d.float()).cpu())
    e.model._layer_hook = hook
    e.step([("a", ids)])
    for i, (a, b) in enumerate(zip(got, want)):
        assert float(lu.row_errors(a, b).max()) < TOL[dtype], i


@pytest.mark.parametrize("name", ["small", "uneven", "wide"])
@pytest.mark.parametrize("dtype", [F32, BF])
def test_ragged_batches_equal_each_alone(models, name, dtype):
    """Prompts of unequal lengths in one batch, decoded together with sequences that end earlier; then other sequences in the
    freed slots and pages, admitted while some are still decoding."""
    folder, ref = models[name]
    V = CFG[name]["vocab"]
    lens = [1, 2, 47, 48, 49, 130, 257]
    seqs = [lu.tokens(n + 30, V, 100 + n) for n in lens]
    want = [ref.logits(s) for s in seqs]
    e = engine(folder, dtype, slots=7, pages=16)
    poison(e)

    def check(k, lo, got):
        err = lu.row_errors(got.float(), want[k][lo:lo + got.shape[0]])
        assert float(err.max()) < TOL[dtype], (name, k, lo, float(err.max()))
    _, lg = e.step([(k, s[:n]) for k, (s, n) in enumerate(zip(seqs, lens))], [list(range(n)) for n in lens], sample=False)
    at = 0
    for k, n in enumerate(lens):
        check(k, 0, lg[at:at + n])
        at += n
    live = list(range(len(lens)))
    for t in range(30):
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


@pytest.mark.parametrize("dtype", [F32, BF])
def test_logits_do_not_depend_on_the_batch(models, dtype):
    """The same sequence alone, in a batch, in other slots: equal up to the GEMMs' own dependence on the number of rows."""
    folder, _ = models["wide"]
    seqs = [lu.tokens(n, 512, n) for n in (70, 33, 201)]
    e = engine(folder, dtype, slots=4, pages=12)
    alone = []
    for s in seqs:
        alone.append(e.step([("x", s)], [[len(s) - 1]], sample=False)[1])
        e.end("x")
    _, together = e.step([(k, s) for k, s in enumerate(seqs)], [[len(s) - 1] for s in seqs], sample=False)
    err = lu.row_errors(together.float(), torch.cat(alone).double().cpu())
    assert float(err.max()) < TOL[dtype] / 2


def test_long_decoding_crosses_pages_and_chunks(models):
    folder, ref = models["small"]
    ids = lu.tokens(700, 320, 3)
    want = ref.logits(ids)
    e = engine(folder, F32, slots=1)
    got = feed(e, "a", ids, [3] + [1] * 697)
    assert float(lu.row_errors(got, want).max()) < TOL[F32]


def test_far_keys_show(tmp_path):
    """One layer whose query projection maps token t to the key of token t + 32: a token asks for ONE earlier token, at its
    chunk's first position, from the chunk's last, or one position outside the chunk."""
    W, V, chunk = 128, 64, 100
    cfg = lu.config([lu.layer(heads=2, kv_heads=1, dim=128, vdim=64, chunk=chunk, scale=12.0 / 128, ff=64)], vocab=V, width=W)
    t = lu.tensors(cfg, 2)
    t["pos"] *= 0.02
    t["l0.shift"] *= 0.1
    t["l0.norm1"].fill_(1.0)
    t["l0.mix.o"] *= 6
    E = lr.rms(t["embed"].double(), 1e-5)
    asks = (torch.linalg.pinv(E) @ E.roll(-32, 0)).T              # asks @ E[t] = E[t + 32]
    t["l0.mix.q"], t["l0.mix.k"] = torch.cat([asks, asks]).to(BF), torch.eye(W).to(BF)
    folder, ref = lu.write_model(tmp_path / "far", cfg, t), lr.RefModel(cfg, t)
    ids = [1 + i % 20 for i in range(300)]
    for x, (j, i) in enumerate(((0, 98), (100, 199), (99, 150), (99, 101), (200, 299), (198, 202), (197, 290)), 21):
        ids[i] = x
        ids[j] = x + 32 if ids[j] < 53 else ids[j]
        if ids[j] != x + 32:
            ids[i] = ids[j] - 32
    want = ref.logits(ids)
    for dtype in (F32, BF):
        e = engine(folder, dtype, slots=1)
        for label, cuts in (("w", [300]), ("d", [98] + [1] * 202)):
            assert float(lu.row_errors(feed(e, label, ids, cuts), want).max()) < TOL[dtype], (dtype, label)
            e.end(label)
    real = lr.attention
    try:                                               # a mask one token off would show
        for by in (-1, 1):
            lr.attention = lambda q, k, v, r1, r2, s, c, eps, p=0: real(q, k, v, r1, r2, s, c + by, eps, p)
            assert float(lu.row_errors(ref.logits(ids), want).max()) > 10 * TOL[BF]
    finally:
        lr.attention = real


def greedy_close(ref, prompt, got, gap=0.05):
    """`got` is the greedy continuation, up to steps where the two best logits nearly tie."""
    st = ref.new_state()
    lg = ref.step(torch.tensor(prompt), st)[-1]
    spread = float(lg.std())
    for t in got:
        best = float(lg.max())
        assert best - float(lg[t]) <= gap * spread, (t, int(lg.argmax()), best, float(lg[t]))
        lg = ref.step(torch.tensor([t]), st)[-1]


@pytest.mark.parametrize("name", ["small", "uneven", "wide"])
@pytest.mark.parametrize("graphs", [False, True])
def test_greedy_generation_through_the_engine(models, name, graphs):
    """encode + inference of a fixed batch (the baseline loop), eager and with captured decode steps, twice over the same
    engine; decoding crosses pages."""
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
        out, steps, _ = harness.run_baseline_batch(e, prompts, 165, -1, -1)
        assert out.shape == (3, 165) and steps == 43
        for b in range(3):
            greedy_close(ref, prompts[b].tolist(), out[b, 121:].tolist())
        if trial == 0:
            first = out
    assert not torch.equal(first, out)


@pytest.mark.parametrize("dtype", [F32, BF])
def test_continuous_batching(models, dtype):
    """More prompts of unequal lengths than slots, with an end token: sequences come and go; in 32-bit the tokens are those of
    the plain implementation."""
    from magicdec_amd import harness
    folder, ref = models["small"]
    prompts = [lu.tokens(n, 320, 900 + n) for n in (5, 130, 1, 64, 260, 33, 128)]
    e = engine(folder, dtype, slots=3, pages=7)
    out, steps, _ = harness.run_sequences(e, prompts, 20, eot=(7,))
    assert not e.pool.seqs and len(e.pool.free_pages) == 7
    for p, o in zip(prompts, out):
        assert len(o) == 20 or o[-1] == 7
        greedy_close(ref, p, o, 0.05 if dtype == BF else 1e-3)
    with pytest.raises(ValueError, match="does not fit"):
        harness.run_sequences(e, [[1] * 900], 100)


def test_speculative_decoding_with_a_draft_of_the_design(models):
    """The longspec loop with this design as target and as (full-cache) draft: the draft is the target, every token is
    accepted, rejected tails roll the state back, and the output is the greedy one."""
    from magicdec_amd import harness
    from magicdec_amd.Engine.SnapKV.backend import LMBackend
    from magicdec_amd.Engine.SnapKV.backend_draft import LMBackend_Draft
    folder, ref = models["small"]
    other = models["wide"][0]
    gamma = 3
    prompts = torch.tensor([lu.tokens(121, 320, 40 + b) for b in range(2)], device=DEV)
    e = LMBackend(dtype=BF, device=DEV, dec_len=gamma + 1)
    e.load_model(folder, use_tp=False)
    e.setup_caches(max_batch_size=2, max_seq_length=256)
    d = LMBackend_Draft(dtype=BF, device=DEV, draft_budget=-1)
    d.load_model(folder, use_tp=False)
    d.setup_caches(max_batch_size=2, max_seq_length=256, draft_budget=-1)
    for forced in (None, lambda st: torch.tensor([2, 1], device=DEV)):
        st, _ = harness.run_longspec_batch(e, d, prompts, gamma, 250, -1, -1, forced_accept_fn=forced)
        assert int(st.num_nodes.max()) >= 121 + 60 and int(st.num_nodes.min()) >= 121 + 30
        if forced is None:
            for b in range(2):
                greedy_close(ref, prompts[b].tolist(), st.output[b, 121:int(st.num_nodes[b])].tolist())
    with pytest.raises(ValueError, match="take back"):
        harness.run_longspec_batch(e, d, prompts, 20, 250, -1, -1)
    s = LMBackend_Draft(dtype=BF, device=DEV, draft_budget=129)
    s.load_model(other, use_tp=False)
    with pytest.raises(NotImplementedError):
        s.setup_caches(max_batch_size=2, max_seq_length=256, draft_budget=129)


def test_rolled_back_tokens_leave_no_trace(models):
    """Verify steps of four tokens of which one or two are kept: the logits are those of the kept sequence."""
    from magicdec_amd.Engine.SnapKV.backend import LMBackend
    folder, ref = models["wide"]
    e = LMBackend(dtype=BF, device=DEV, dec_len=4)
    e.load_model(folder, use_tp=False)
    e.setup_caches(max_batch_size=2, max_seq_length=300)
    seqs = [lu.tokens(200, 512, b) for b in (1, 2)]
    want = [ref.logits(s) for s in seqs]
    e.encode(torch.tensor([s[:120] for s in seqs], device=DEV))
    at = [120, 120]
    for step in range(20):
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
    steps += [{"step": 3 + i, "entries": [{"id": "b", "tokens": seqs["b"][6 + i:7 + i], "want": [0]}], "end": ["b"] if i == 2 else []}
              for i in range(3)]
    p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", dtype, "--out", str(tmp_path),
                        "--max-tokens", "160"], input="".join(json.dumps(s) + "\n" for s in steps), text=True,
                       capture_output=True, timeout=110)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [ln for ln in p.stdout.splitlines() if ln.startswith("done")] == [f"done {i}" for i in range(6)]
    assert not (tmp_path / "1.f32").exists()
    expect = {0: [("a", 139), ("a", 0), ("a", 70)], 2: [("c", 60), ("b", 5)], 3: [("b", 6)], 4: [("b", 7)], 5: [("b", 8)]}
    for s, rows in expect.items():
        got = torch.frombuffer(bytearray((tmp_path / f"{s}.f32").read_bytes()), dtype=F32).view(len(rows), 211)
        ref_rows = torch.stack([want[k][i] for k, i in rows])
        assert float(lu.row_errors(got, ref_rows).max()) < TOL[getattr(torch, dtype)] * 1.5, s


def test_command_line_serves_the_design(models, capsys):
    """The baseline command line over a checkpoint folder, fixed batch and ragged."""
    from magicdec_amd import cli
    folder = models["small"][0]
    base = ["--model", folder, "--rank_group", "0", "--B", "2", "--prefix_len", "100", "--max_len", "128"]
    assert cli.baseline_main(base) > 0
    assert cli.baseline_main(base + ["--ragged", "--dtype", "float32"]) > 0
    assert "sequences :20" in capsys.readouterr().out


def test_llama_checkpoints_serve_ragged_steps():
    """The same step() over a Llama-style model of the zoo: unequal sequences equal each alone."""
    from pathlib import Path
    from magicdec_amd.Engine import model_core
    from magicdec_amd.Engine.SnapKV.backend import LMBackend
    model_core.transformer_configs["raggedtiny"] = dict(block_size=2048, n_layer=2, n_head=8, n_local_heads=2, dim=512,
                                                        intermediate_size=1024, vocab_size=1000)
    e = LMBackend(dtype=BF, device=DEV)
    e.load_model(Path("/nonexistent/raggedtiny/model.pth"), use_tp=False)
    e.setup_caches(max_batch_size=3, max_seq_length=512)
    seqs = [lu.tokens(n + 6, 1000, n) for n in (40, 131, 3)]
    alone = []
    for s in seqs:
        _, lg = e.step([("x", s)], [list(range(len(s)))], sample=False)
        alone.append(lg.float().cpu())
        e.end("x")
    e.step([(k, s[:-6]) for k, s in enumerate(seqs)], sample=False)
    for t in range(6):
        toks, lg = e.step([(k, [s[len(s) - 6 + t]]) for k, s in enumerate(seqs)], [[0]] * 3)
        for k, s in enumerate(seqs):
            w = alone[k][len(s) - 6 + t]
            assert float((lg[k].float().cpu() - w).abs().max()) < 0.05 * float(w.abs().max())
            assert int(toks[k]) == int(lg[k].argmax())
