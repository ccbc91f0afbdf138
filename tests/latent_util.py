"""Small random models of the latent-attention decoder design for the tests: a config.json, a model.safetensors (bfloat16) and the
plain implementation (oracle/latent_ref.py) of the same weights."""
import torch

from oracle import latent_ref as la
from tests.layers_util import row_errors, tokens, write_model  # noqa: F401  (the tests' common helpers)

YARN = {"factor": 5.0, "original": 96, "fast": 6.0, "slow": 0.5}


def layer(kind=1, heads=4, dim=24, rot_dim=8, vdim=40, q_rank=56, kv_rank=48, ff=136, scale=None, base=700.0, yarn=None, kv_from=None,
          mlp=True):
    """kind 1: gated heads; kind 2: no gate, YaRN (unless yarn is None), optionally another layer's cache."""
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
         "scale": (dim + rot_dim) ** -0.5 if scale is None else scale, "rot": {"dims": rot_dim, "base": base}}
    if yarn is not None:
        m["rot"]["scaling"] = dict(yarn)
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention" if kind == 1 else "latent_attention_2", "mixer": m,
            "mlp": {"kind": "dense", "ff": ff} if mlp else None}


def config(layers, vocab=300, width=120, eps=1e-5, softcap=12.0, buckets=509, mul_prev=131, mul_cur=17):
    return {"architecture": "Bufodra", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_softcap": softcap,
            "embedding": {"bigram": {"buckets": buckets, "mul_prev": mul_prev, "mul_cur": mul_cur}}, "layers": layers}


def tensors(cfg, seed, gain=1.0, bf16=True):
    """Random weights; norms differ from 1, gates from one half."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]

    def lin(o, i, s=1.0):
        return torch.randn(o, i, generator=g) * (s * gain / i ** 0.5)

    def around(n):
        return 1.0 + 0.4 * (2 * torch.rand(n, generator=g) - 1)
    t = {"embed": torch.randn(V, W, generator=g) * 0.5, "bigram": torch.randn(cfg["embedding"]["bigram"]["buckets"] + 1, W, generator=g) * 0.5,
         "embed.norm": around(W), "final.norm": around(W)}
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        H, D, RD, VD, Q, R = (m[k] for k in ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank"))
        t[p + "norm1"] = around(W)
        t[p + "mix.dq"], t[p + "mix.dq.norm"], t[p + "mix.uq"] = lin(Q, W), around(Q), lin(H * (D + RD), Q, 1.6)
        if m.get("kv_from") is None:
            t[p + "mix.dkv"], t[p + "mix.dkv.norm"] = lin(R + RD, W), around(R)
        t[p + "mix.uk"], t[p + "mix.uv"], t[p + "mix.o"] = lin(H * D, R, 1.6), lin(H * VD, R), lin(W, H * VD)
        if L["type"] == "latent_attention":
            t[p + "mix.g"] = lin(H, W, 1.5)
        if L["mlp"] is not None:
            ff = L["mlp"]["ff"]
            t[p + "mlp.gate"], t[p + "mlp.up"], t[p + "mlp.down"] = lin(ff, W, 1.5), lin(ff, W), lin(W, ff)
    return {k: v.to(torch.bfloat16) if bf16 else v for k, v in t.items()}


def make(folder, cfg, seed, gain=1.0):
    """(folder, plain implementation)"""
    t = tensors(cfg, seed, gain)
    return write_model(folder, cfg, t), la.LatentRefModel(cfg, t)


def asking_model(seed=3, vocab=64, width=128, heads=2, score=16.0, n=300, shift=32, borders=()):
    """A one-layer model whose token t (t < shift) asks for token t + shift, and a sequence of `n` filler tokens with
    `borders` = (asked-for place, asking place) pairs in it.  -> (cfg, tensors, ids)"""
    dim = 64
    cfg = config([layer(1, heads=heads, dim=dim, rot_dim=16, vdim=48, q_rank=width, kv_rank=width, ff=64, scale=score / dim)], vocab=vocab,
                 width=width)
    t = {k: v.float() for k, v in tensors(cfg, seed).items()}
    t["bigram"] *= 0.02
    for k in ("embed.norm", "l0.norm1", "l0.mix.dq.norm", "l0.mix.dkv.norm"):
        t[k].fill_(1.0)
    E = t["embed"] / t["embed"].pow(2).mean(-1, keepdim=True).sqrt()
    asks = (torch.linalg.pinv(E.double()) @ E.double().roll(-shift, 0)).T.float()          # asks @ E[t] = E[t + shift]
    P = torch.linalg.qr(torch.randn(width, dim, generator=torch.Generator().manual_seed(seed)))[0].T
    t["l0.mix.dq"] = asks
    t["l0.mix.dkv"][:width], t["l0.mix.dkv"][width:] = torch.eye(width), 0.05 * t["l0.mix.dkv"][width:]
    uq = t["l0.mix.uq"].view(heads, dim + 16, width)
    uq[:, :dim], uq[:, dim:] = P, 0.05 * uq[:, dim:]
    t["l0.mix.uk"] = P.repeat(heads, 1)
    t["l0.mix.o"] *= 6
    ids = [1 + i % (shift // 2 - 2) for i in range(n)]
    for x, (j, i) in enumerate(borders, shift // 2):
        ids[i], ids[j] = x, x + shift
    return cfg, {k: v.to(torch.bfloat16).contiguous() for k, v in t.items()}, ids
