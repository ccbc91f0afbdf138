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
from typing import Optional, Tuple, Union


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
class YarnSpec:
    """YaRN scaling of rotary frequencies (ops.RotaryTable)."""
    factor: float
    original: float
    fast: float
    slow: float


@dataclass(frozen=True)
class RotarySpec:
    """Rotary positions on neighbouring pairs of the first `dims` elements."""
    dims: int
    base: float
    yarn: Optional[YarnSpec] = None


@dataclass(frozen=True)
class LatentAttentionSpec:
    """Softmax attention whose keys and values are linear maps of one latent row per token, beside one rotated key part that all
    heads share; queries come through a latent of their own (ops.LatentSpec holds the same numbers for the kernels)."""
    heads: int
    dim: int                      # unrotated query / key size per head
    rot_dim: int                  # rotated query / key size per head
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rotary: RotarySpec
    gate: bool = False            # a head's output is multiplied by the sigmoid of its own logit
    kv_from: Optional[int] = None   # layer whose cache rows this layer attends to; None: its own


@dataclass(frozen=True)
class MLPSpec:
    ff: int
    act: str = "xielu"            # "xielu": down . act(up . h);  "gelu_gated": down . (gelu_tanh(gate . h) * (up . h))


@dataclass(frozen=True)
class BigramSpec:
    """A second embedding, of the pair (token before, token): row (mul_before * before + mul_token * token) mod buckets."""
    buckets: int
    mul_before: int
    mul_token: int


@dataclass(frozen=True)
class LayerSpec:
    attention: Union[AttentionSpec, LatentAttentionSpec]
    mlp: Optional[MLPSpec]
    token_shift: bool = False
    parallel: bool = False        # mixer and feed-forward read one norm and are added together


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
    bigram: Optional[BigramSpec] = None
    embed_norm: bool = False      # weighted norm behind the embedding
    tied_head: bool = False       # the embedding table is the output head
    logit_softcap: Optional[float] = None

    @property
    def n_layer(self):
        return len(self.layers)


class _Reader:
    """Reads every key of a JSON object exactly once; keys nobody asked for are an error, not silently ignored."""

    def __init__(self, obj, where):
        if not isinstance(obj, dict):
            raise ValueError(f"config.json: {where} must be an object, got {obj!r}")
        self.obj, self.where, self.seen = obj, where, set()

    def has(self, key):
        return self.obj.get(key) is not None

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

    def skip(self, key):
        """An optional key that may be present as null."""
        self.seen.add(key)

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


def _rotary(r: _Reader) -> RotarySpec:
    dims, base, yarn = r.get("dims", int), r.get("base", float), None
    r.skip("scaling")
    if r.has("scaling"):
        s = r.sub("scaling")
        yarn = YarnSpec(*(s.get(k, float) for k in ("factor", "original", "fast", "slow")))
        s.done()
    r.done()
    if dims % 2:
        raise ValueError(f"config.json: {r.where}.dims must be even, got {dims}")
    return RotarySpec(dims, base, yarn)


def _bufodra(cfg) -> DecoderSpec:
    """Bufodra: parallel layers (latent attention beside a gated GELU feed-forward, one norm); of the two kinds of mixer one gates
    its heads, the other may attend to an earlier layer's cache; a bigram embedding under a norm, a tied head, a logit soft cap."""
    c = _Reader(cfg, "the model")
    c.get("architecture")
    norm, emb = c.sub("norm"), c.sub("embedding")
    big = emb.sub("bigram")
    bigram = BigramSpec(buckets=big.get("buckets", int), mul_before=big.get("mul_prev"), mul_token=big.get("mul_cur"))
    if not all(isinstance(v, int) and not isinstance(v, bool) for v in (bigram.mul_before, bigram.mul_token)):
        raise ValueError("config.json: the bigram's multipliers must be integers")
    layers = []
    for i, obj in enumerate(c.get("layers")):
        L = _Reader(obj, f"layers[{i}]")
        kind = L.get("type")
        if kind not in ("latent_attention", "latent_attention_2"):
            raise ValueError(f"config.json: layers[{i}]: unknown mixer {kind!r}")
        m = L.sub("mixer")
        m.skip("kv_from")
        att = LatentAttentionSpec(heads=m.get("heads", int), dim=m.get("dim", int), rot_dim=m.get("rot_dim", int),
                                  vdim=m.get("vdim", int), q_rank=m.get("q_rank", int), kv_rank=m.get("kv_rank", int),
                                  scale=m.get("scale", float), rotary=_rotary(m.sub("rot")), gate=kind == "latent_attention",
                                  kv_from=m.get("kv_from") if m.has("kv_from") else None)
        m.done()
        if att.rotary.dims > att.rot_dim:
            raise ValueError(f"config.json: layers[{i}]: {att.rotary.dims} rotated dimensions of {att.rot_dim}")
        if att.kv_from is not None:
            src = layers[att.kv_from].attention if isinstance(att.kv_from, int) and 0 <= att.kv_from < i else None
            if src is None or src.kv_from is not None or (src.kv_rank, src.rot_dim, src.rotary) != (att.kv_rank, att.rot_dim, att.rotary):
                raise ValueError(f"config.json: layers[{i}]: kv_from must name an earlier layer with a cache of its own and the same "
                                 "kv_rank, rot_dim and rotation")
        mlp = None
        if L.get("mlp") is not None:
            f = L.sub("mlp")
            if f.get("kind") != "dense":
                raise ValueError(f"config.json: layers[{i}]: unknown feed-forward {f.obj['kind']!r}")
            mlp = MLPSpec(ff=f.get("ff", int), act="gelu_gated")
            f.done()
        L.done()
        layers.append(LayerSpec(attention=att, mlp=mlp, parallel=True))
    spec = DecoderSpec(design="Bufodra", vocab_size=c.get("vocab", int), dim=c.get("width", int), norm_eps=norm.get("eps", float),
                       layers=tuple(layers), bigram=bigram, embed_norm=True, tied_head=True,
                       logit_softcap=c.get("logit_softcap", float))
    for r in (norm, big, emb, c):
        r.done()
    if not layers:
        raise ValueError("config.json: the model has no layers")
    if not spec.logit_softcap > 0:
        raise ValueError("config.json: logit_softcap must be positive")
    return spec


DESIGNS = {"Furitar": _furitar, "Bufodra": _bufodra}


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


def _bufodra_config(vocab, width, n_layer, heads, dim, rot_dim, vdim, q_rank, kv_rank, ff, original=4096):
    """Pairs of a gated layer and a YaRN layer; every second YaRN layer attends to the cache of the one before it."""
    def layer(i):
        mixer = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
                 "scale": (dim + rot_dim) ** -0.5, "rot": {"base": 10000.0, "dims": rot_dim}}
        if i % 2:
            mixer["rot"] = dict(mixer["rot"], scaling={"factor": 8.0, "original": original, "fast": 32.0, "slow": 1.0})
            if i % 4 == 3:
                mixer["kv_from"] = i - 2
        return {"type": "latent_attention_2" if i % 2 else "latent_attention", "mixer": mixer, "mlp": {"kind": "dense", "ff": ff}}
    return {"architecture": "Bufodra", "vocab": vocab, "width": width, "norm": {"eps": 1e-5}, "logit_softcap": 30.0,
            "embedding": {"bigram": {"buckets": 65536, "mul_prev": 31337, "mul_cur": 7919}}, "layers": [layer(i) for i in range(n_layer)]}


# named configurations of the designs (random weights where no checkpoint exists): the widths of the model zoo's
# Llama-3.2-1B and Llama-3.1-8B, so that the two families can be measured side by side
design_configs = {
    "furitar-1b": _furitar_config(128256, 2048, 16, 32, 8, 64, 64, 8192, 8192, 32768),
    "furitar-8b": _furitar_config(128256, 4096, 32, 32, 8, 128, 128, 14336, 8192, 32768),
    "bufodra-1b": _bufodra_config(128256, 2048, 16, 16, 128, 64, 128, 768, 512, 5632),
    "bufodra-8b": _bufodra_config(128256, 4096, 32, 32, 128, 64, 128, 1536, 512, 12288),
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
