"""Registry of the decoder designs that are described layer by layer (a config.json next to model.safetensors) instead of by
a Llama-style ModelArgs.

A design is a reader of its config.json: it returns a `DecoderSpec`, plain data that says which mechanisms every layer has and
with which constants.  The model (Engine/model_layers.py), its caches and its kernels know the mechanisms only, so another
design that combines them differently is another reader here.
"""
from __future__ import annotations

import json
from dataclasses import dataclass
from pathlib import Path
from typing import Optional, Tuple


@dataclass(frozen=True)
class AttentionSpec:
    """Softmax attention over a paged cache (ops.XattnSpec holds the same numbers for the kernels)."""
    heads: int
    kv_heads: int
    dim: int                      # query / key size per head
    vdim: int                     # value size per head
    scale: float
    chunk: int = 0                # positions see their own chunk only; 0: no chunks
    qk_norm: bool = False         # query and key heads scaled to unit RMS, without weights
    distance_bias: bool = False   # logarithmic penalty on the distance, two coefficients per head
    sink: bool = False            # the softmax leaves weight 1 / (1 + S) unassigned (S: the sum of the exponentials)


@dataclass(frozen=True)
class MLPSpec:
    ff: int
    act: str = "xielu"


@dataclass(frozen=True)
class LayerSpec:
    attention: AttentionSpec
    mlp: Optional[MLPSpec]
    token_shift: bool = False


@dataclass(frozen=True)
class DecoderSpec:
    design: str
    vocab_size: int
    dim: int                      # width of the residual stream
    norm_eps: float
    layers: Tuple[LayerSpec, ...]
    embed_scale: float = 1.0
    logit_scale: float = 1.0
    max_positions: int = 0        # learned position vectors; 0: none

    @property
    def n_layer(self):
        return len(self.layers)


class _Reader:
    """Reads every key of a JSON object exactly once; keys nobody asked for are an error, not silently ignored."""

    def __init__(self, obj, where):
        if not isinstance(obj, dict):
            raise ValueError(f"config.json: {where} must be an object, got {obj!r}")
        self.obj, self.where, self.seen = obj, where, set()

    def get(self, key, kind=None):
        if key not in self.obj:
            raise ValueError(f"config.json: {self.where} has no '{key}'")
        self.seen.add(key)
        v = self.obj[key]
        if kind is int and (isinstance(v, bool) or not isinstance(v, int) or v <= 0):
            raise ValueError(f"config.json: {self.where}.{key} must be a positive integer, got {v!r}")
        if kind is float:
            if isinstance(v, bool) or not isinstance(v, (int, float)):
                raise ValueError(f"config.json: {self.where}.{key} must be a number, got {v!r}")
            v = float(v)
        return v

    def sub(self, key):
        return _Reader(self.get(key), f"{self.where}.{key}")

    def done(self):
        extra = sorted(set(self.obj) - self.seen)
        if extra:
            raise ValueError(f"config.json: {self.where}: unknown keys {extra}")


def _furitar(cfg) -> DecoderSpec:
    """Furitar: pre-norm layers with a token shift in front of every mixer; chunked softmax attention with unit-RMS queries and keys, a
    logarithmic distance penalty and a sink; learned positions; dense xIELU feed-forwards (or none)."""
    c = _Reader(cfg, "the model")
    c.get("architecture")
    emb, norm = c.sub("embedding"), c.sub("norm")
    layers = []
    for i, obj in enumerate(c.get("layers")):
        L = _Reader(obj, f"layers[{i}]")
        if L.get("type") != "attention":
            raise ValueError(f"config.json: layers[{i}]: unknown mixer {obj['type']!r}")
        m = L.sub("mixer")
        mask = m.sub("mask")
        att = AttentionSpec(heads=m.get("heads", int), kv_heads=m.get("kv_heads", int), dim=m.get("dim", int),
                            vdim=m.get("vdim", int), scale=m.get("scale", float), chunk=mask.get("size", int),
                            qk_norm=True, distance_bias=True, sink=True)
        mask.done()
        m.done()
        if att.heads % att.kv_heads:
            raise ValueError(f"config.json: layers[{i}]: {att.heads} heads do not share {att.kv_heads} kv heads evenly")
        mlp = None
        if L.get("mlp") is not None:
            f = L.sub("mlp")
            if f.get("kind") != "dense":
                raise ValueError(f"config.json: layers[{i}]: unknown feed-forward {f.obj['kind']!r}")
            mlp = MLPSpec(ff=f.get("ff", int), act="xielu")
            f.done()
        L.done()
        layers.append(LayerSpec(attention=att, mlp=mlp, token_shift=True))
    spec = DecoderSpec(design="Furitar", vocab_size=c.get("vocab", int), dim=c.get("width", int),
                       norm_eps=norm.get("eps", float), layers=tuple(layers), embed_scale=emb.get("scale", float),
                       logit_scale=c.get("logit_scale", float), max_positions=c.get("max_positions", int))
    for r in (emb, norm, c):
        r.done()
    if not layers:
        raise ValueError("config.json: the model has no layers")
    return spec


DESIGNS = {"Furitar": _furitar}


def spec_from_config(cfg) -> DecoderSpec:
    name = cfg.get("architecture")
    if name not in DESIGNS:
        raise ValueError(f"config.json: unknown architecture {name!r} (known: {', '.join(DESIGNS)})")
    return DESIGNS[name](cfg)


def _furitar_config(vocab, width, n_layer, heads, kv_heads, dim, vdim, ff, chunk, max_positions):
    layer = {"type": "attention", "mlp": {"kind": "dense", "ff": ff},
             "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5,
                       "mask": {"size": chunk}}}
    return {"architecture": "Furitar", "vocab": vocab, "width": width, "norm": {"eps": 1e-5}, "embedding": {"scale": 1.0},
            "logit_scale": 1.0, "max_positions": max_positions, "layers": [layer] * n_layer}


# named configurations of the designs (random weights where no checkpoint exists): the widths of the model zoo's
# Llama-3.2-1B and Llama-3.1-8B, so that the two families can be measured side by side
design_configs = {
    "furitar-1b": _furitar_config(128256, 2048, 16, 32, 8, 64, 64, 8192, 8192, 32768),
    "furitar-8b": _furitar_config(128256, 4096, 32, 32, 8, 128, 128, 14336, 8192, 32768),
}


def config_path(checkpoint_path) -> Optional[Path]:
    """The config.json that belongs to a checkpoint: of the folder itself, or next to the file."""
    p = Path(checkpoint_path)
    for cand in ((p / "config.json",) if p.is_dir() else (p.parent / "config.json",)):
        if cand.is_file():
            return cand
    return None


def find_design(checkpoint_path) -> Optional[DecoderSpec]:
    """The design a checkpoint path names, or None (the path is a Llama-style checkpoint): by the `architecture` of its
    config.json, else -- no config.json -- by a named configuration contained in its directory name."""
    cfg_file = config_path(checkpoint_path)
    if cfg_file is not None:
        with open(cfg_file) as f:
            cfg = json.load(f)
        return spec_from_config(cfg) if "architecture" in cfg else None
    p = Path(checkpoint_path)
    name = (p.name if p.is_dir() or p.suffix == "" else p.parent.name).lower()
    hits = sorted((k for k in design_configs if k in name), key=len, reverse=True)
    return spec_from_config(design_configs[hits[0]]) if hits else None
