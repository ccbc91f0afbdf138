"""Small random models of the layered decoder designs for the tests: a config.json, a model.safetensors (bfloat16) and the
plain implementation (oracle/layered_ref.py) of the same weights."""
import json
import os

import torch

from oracle import layered_ref as lr


def layer(heads=4, kv_heads=2, dim=32, vdim=32, ff=128, chunk=48, scale=None, mlp=True):
    return {"type": "attention", "mlp": {"kind": "dense", "ff": ff} if mlp else None,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                      "scale": dim ** -0.5 if scale is None else scale, "mask": {"size": chunk}}}


def config(layers, vocab=320, width=128, max_positions=1024, eps=1e-5, embed_scale=1.0, logit_scale=1.0):
    return {"architecture": "Furitar", "vocab": vocab, "width": width, "max_positions": max_positions, "norm": {"eps": eps},
            "embedding": {"scale": embed_scale}, "logit_scale": logit_scale, "layers": layers}


def tensors(cfg, seed, gain=1.0, bf16=True):
    """Random weights; norms, shifts, bias coefficients and activation numbers all differ from their neutral values."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]

    def lin(o, i, s=1.0):
        return torch.randn(o, i, generator=g) * (s * gain / i ** 0.5)

    def around(n, mid, spread):
        return mid + spread * (2 * torch.rand(n, generator=g) - 1)
    t = {"embed": torch.randn(V, W, generator=g), "pos": 0.5 * torch.randn(cfg["max_positions"], W, generator=g),
         "final.norm": around(W, 1.0, 0.4), "head": lin(V, W)}
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        H, G, D, VD = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        t[p + "norm1"], t[p + "shift"] = around(W, 1.0, 0.4), around(W, 0.4, 0.4)
        t[p + "mix.q"], t[p + "mix.k"], t[p + "mix.v"] = lin(H * D, W), lin(G * D, W), lin(G * VD, W)
        t[p + "mix.o"] = lin(W, H * VD)
        t[p + "mix.r1"], t[p + "mix.r2"] = around(H, 0.6, 0.5), around(H, 0.3, 0.25)
        if L["mlp"] is not None:
            t[p + "norm2"] = around(W, 1.0, 0.4)
            t[p + "mlp.up"], t[p + "mlp.down"] = lin(L["mlp"]["ff"], W), lin(W, L["mlp"]["ff"])
            t[p + "mlp.act"] = around(2, 0.1, 0.6)
    return {k: v.to(torch.bfloat16) if bf16 else v for k, v in t.items()}


def write_model(folder, cfg, t):
    from safetensors.torch import save_file
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in t.items()}, os.path.join(folder, "model.safetensors"))
    return str(folder)


def make(folder, cfg, seed, gain=1.0):
    """(folder, plain implementation)"""
    t = tensors(cfg, seed, gain)
    return write_model(folder, cfg, t), lr.RefModel(cfg, t)


def tokens(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def row_errors(got, want):
    """Root mean square of every row's difference over the root mean square of the whole expectation (means taken off)."""
    d = got.double().cpu() - want.double()
    d = d - d.mean(-1, keepdim=True)
    w = want.double() - want.double().mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / w.pow(2).mean().sqrt()
