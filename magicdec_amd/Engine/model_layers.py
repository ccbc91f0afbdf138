"""The layered decoder: one model class for every design of Engine/designs.py.

It is a `Transformer` whose layers follow a `DecoderSpec`: the same step interface (prefill / forward over a page table and
device-side positions, token ids out), weight packing, GEMM policy, graph capture and back-ends; what differs is what a layer
computes:

* the residual stream is float32; the residual add, the RMS norm behind it and the token shift are one launch
  (ops.resid_norm), fed by the projection's 16-bit rows or directly by a split-K product's float32 planes;
* attention is ops.extended_attention: separate query/key and value head sizes, query/key norm, distance bias, chunk mask and
  sink, over `SplitKVCache` pages that are addressed by position; decode steps normalise, append and attend in one launch;
* latent attention (ops.latent_append, ops.latent_attention) keeps one `LatentCache` row per token for all heads; layers may
  share another layer's cache.  A parallel layer is two products in (mixer; gate and up) and one out: head outputs and
  activations are written side by side and meet one [wo | down] matrix;
* a bigram embedding reads the token before from a paged token history (ops.embed_bigram);
* the last unshifted rows of every sequence live in a small float32 ring per layer, indexed by position (ops.resid_norm), so a
  step may be repeated (graph capture) or rolled back (rejected draft tokens) without saving state.

With float32 weights every kernel runs in 32-bit (plain attention kernel, library GEMMs without reduced-precision modes).
"""
from __future__ import annotations

import math

import torch
import torch.nn as nn
from torch.nn import functional as F

from .. import ops
from .designs import DecoderSpec, LatentAttentionSpec, LayerSpec
from .gemm_policy import choose, use_split
from .model_core import PageTable, RMSNorm, Transformer

STATE_RING = 16        # unshifted rows kept per sequence and layer: rollbacks of up to STATE_RING - 2 tokens


class SplitKVCache(nn.Module):
    """Paged keys [pages, KH, page_size, pad(D)] and values [pages, KH, page_size, pad(DV)] of one layer.  A page list maps
    every position of its sequence, so stale rows are never read and nothing has to be cleared between sequences."""

    def __init__(self, num_pages, page_size, kv_heads, dim, vdim, dtype):
        super().__init__()
        self.register_buffer("k_cache", torch.zeros((num_pages, kv_heads, page_size, ops.head_pad(dim)), dtype=dtype),
                             persistent=False)
        self.register_buffer("v_cache", torch.zeros((num_pages, kv_heads, page_size, ops.head_pad(vdim)), dtype=dtype),
                             persistent=False)
        self.calibrated = False

    def clear(self):
        pass


class LatentCache(nn.Module):
    """Paged rows [pages, page_size, row width] of one layer (and of the layers that attend to it): latent | rotated key part |
    zeros, addressed by position."""

    def __init__(self, num_pages, page_size, kv_rank, rot_dim, dtype):
        super().__init__()
        self.register_buffer("rows", torch.zeros((num_pages, page_size, ops.latent_row_width(kv_rank, rot_dim)), dtype=dtype),
                             persistent=False)
        self.calibrated = False

    def clear(self):
        pass


class LatentAttention(nn.Module):
    def __init__(self, dim, spec: LatentAttentionSpec):
        super().__init__()
        self.spec, self.own_cache = spec, spec.kv_from is None
        # rows of the product in: query latent | latent | key part | gate logits
        self.cuts = [spec.q_rank, spec.kv_rank + spec.rot_dim if self.own_cache else 0, spec.heads if spec.gate else 0]
        self.win = nn.Linear(dim, sum(self.cuts), bias=False)
        self.dq_norm = RMSNorm(spec.q_rank)
        self.kv_norm = RMSNorm(spec.kv_rank) if self.own_cache else None
        self.wuq = nn.Linear(spec.q_rank, spec.heads * (spec.dim + spec.rot_dim), bias=False)
        self.wukv = nn.Linear(spec.kv_rank, spec.heads * (spec.dim + spec.vdim), bias=False)
        self.kv_cache = None

    def kernel_spec(self, eps, rotary) -> ops.LatentSpec:
        s = self.spec
        return ops.LatentSpec(s.heads, s.dim, s.rot_dim, s.vdim, s.q_rank, s.kv_rank, s.scale, eps, rotary, self.wukv.weight.detach(),
                              self.dq_norm.weight.detach(), self.kv_norm.weight.detach() if self.own_cache else None)


class ExtendedAttention(nn.Module):
    def __init__(self, dim, spec):
        super().__init__()
        self.spec = spec
        self.wqkv = nn.Linear(dim, (spec.heads + spec.kv_heads) * spec.dim + spec.kv_heads * spec.vdim, bias=False)
        self.wo = nn.Linear(spec.heads * spec.vdim, dim, bias=False)
        if spec.distance_bias:
            self.r1 = nn.Parameter(torch.empty(spec.heads))
            self.r2 = nn.Parameter(torch.empty(spec.heads))
        self.kv_cache = None

    def kernel_spec(self, eps, max_positions) -> ops.XattnSpec:
        """The layer's constants for the kernels, with the bound on its scores that the matrix-core kernels rely on:
        normalised queries and keys have |q.k| <= D, and a bias with r1 < 0 adds at most |r1| ln(1 + r2 * distance)."""
        s = self.spec
        r1 = r2 = None
        bound = 1.02 * s.dim * abs(s.scale) if s.qk_norm else 0.0        # 2 %: the 16-bit rounding of q and k
        if s.distance_bias:
            r1, r2 = self.r1.detach().float().contiguous(), self.r2.detach().float().contiguous()
            reach = (min(s.chunk, max_positions) if s.chunk else max_positions) - 1
            a, b = r1.double().cpu(), r2.double().cpu()
            if bool((b < 0).any()) or not bool(torch.isfinite(a).all() and torch.isfinite(b).all()):
                bound = 0.0
            elif bound > 0:
                bound += float(((-a).clamp(min=0) * torch.log1p(b * reach)).max())
        return ops.XattnSpec(s.heads, s.kv_heads, s.dim, s.vdim, s.scale, eps, s.chunk, s.sink, s.qk_norm, r1, r2, bound)


class DenseMLP(nn.Module):
    """down . act(up . h)"""

    def __init__(self, dim, spec):
        super().__init__()
        if spec.act != "xielu":
            raise ValueError(f"unknown activation {spec.act!r}")
        self.up = nn.Linear(dim, spec.ff, bias=False)
        self.down = nn.Linear(spec.ff, dim, bias=False)
        self.act = nn.Parameter(torch.empty(2))


class ParallelLayer(nn.Module):
    """Mixer and feed-forward of one norm's output: x + wout . (heads | gelu(gate . y) * (up . y))"""

    def __init__(self, dim, eps, spec: LayerSpec):
        super().__init__()
        if not isinstance(spec.attention, LatentAttentionSpec) or spec.token_shift or (spec.mlp and spec.mlp.act != "gelu_gated"):
            raise ValueError("a parallel layer has latent attention and a gated feed-forward (or none)")
        self.attention_norm = RMSNorm(dim, eps)
        self.attention = LatentAttention(dim, spec.attention)
        self.heads_out = spec.attention.heads * spec.attention.vdim
        ff = spec.mlp.ff if spec.mlp is not None else 0
        self.w13 = nn.Linear(dim, 2 * ff, bias=False) if ff else None            # gate, then up
        self.wout = nn.Linear(self.heads_out + ff, dim, bias=False)              # wo | down
        self.feed_forward = None


class DecoderLayer(nn.Module):
    def __init__(self, dim, eps, spec: LayerSpec):
        super().__init__()
        if isinstance(spec.attention, LatentAttentionSpec) or (spec.mlp and spec.mlp.act != "xielu"):
            raise ValueError("a sequential layer has extended attention and an xIELU feed-forward (or none)")
        self.attention_norm = RMSNorm(dim, eps)
        self.attention = ExtendedAttention(dim, spec.attention)
        if spec.token_shift:
            self.shift = nn.Parameter(torch.empty(dim))
        self.feed_forward = None
        if spec.mlp is not None:
            self.ffn_norm = RMSNorm(dim, eps)
            self.feed_forward = DenseMLP(dim, spec.mlp)


class LayeredTransformer(Transformer):
    position_addressed = True        # pages are found by position: the back-end maps a request's whole page list at once

    def __init__(self, spec: DecoderSpec):
        nn.Module.__init__(self)
        self.config = self.spec = spec
        self.tok_embeddings = nn.Embedding(spec.vocab_size, spec.dim)
        self.pos_embeddings = nn.Embedding(spec.max_positions, spec.dim) if spec.max_positions else None
        self.pair_embeddings = nn.Embedding(spec.bigram.buckets + 1, spec.dim) if spec.bigram else None
        if bool(spec.bigram) != spec.embed_norm or (spec.bigram and spec.max_positions):
            raise ValueError("the embedding is tokens (+ positions), or tokens and pairs under a norm")
        self.embed_norm = RMSNorm(spec.dim, spec.norm_eps) if spec.embed_norm else None
        self.layers = nn.ModuleList((ParallelLayer if s.parallel else DecoderLayer)(spec.dim, spec.norm_eps, s) for s in spec.layers)
        self.norm = RMSNorm(spec.dim, spec.norm_eps)
        self.output = nn.Linear(spec.dim, spec.vocab_size, bias=False)
        self.world_size = self.rank = self.process_group = None
        self._ready, self.skip_head = False, False
        # the expanded form of latent attention computes the context's keys and values anew in every portion: fewer, longer ones
        self.prefill_rows = 65536 if any(s.parallel for s in spec.layers) else 0

    # ------------------------------------------------------------------ weights
    def state_from_tensors(self, t):
        """state_dict of this model from the tensors of a model.safetensors file (embed, pos, l<i>.norm1, l<i>.mix.q, ...)."""
        used = set()

        def take(name):
            used.add(name)
            if name not in t:
                raise KeyError(f"model.safetensors has no tensor '{name}'")
            return t[name]
        sd = {"tok_embeddings.weight": take("embed"), "norm.weight": take("final.norm")}
        sd["output.weight"] = sd["tok_embeddings.weight"] if self.spec.tied_head else take("head")
        if self.pair_embeddings is not None:
            sd["pair_embeddings.weight"] = take("bigram")
        if self.embed_norm is not None:
            sd["embed_norm.weight"] = take("embed.norm")
        if self.pos_embeddings is not None:
            sd["pos_embeddings.weight"] = take("pos")
        for i, s in enumerate(self.spec.layers):
            p, m = f"layers.{i}.", f"l{i}."
            sd[p + "attention_norm.weight"] = take(m + "norm1")
            if s.parallel:
                a = s.attention
                sd[p + "attention.win.weight"] = torch.cat([take(m + "mix.dq")] + ([take(m + "mix.dkv")] if a.kv_from is None else [])
                                                           + ([take(m + "mix.g")] if a.gate else []))
                sd[p + "attention.dq_norm.weight"], sd[p + "attention.wuq.weight"] = take(m + "mix.dq.norm"), take(m + "mix.uq")
                if a.kv_from is None:
                    sd[p + "attention.kv_norm.weight"] = take(m + "mix.dkv.norm")
                sd[p + "attention.wukv.weight"] = torch.cat([take(m + "mix.uk"), take(m + "mix.uv")])
                out = [take(m + "mix.o")]
                if s.mlp is not None:
                    sd[p + "w13.weight"] = torch.cat([take(m + "mlp.gate"), take(m + "mlp.up")])
                    out.append(take(m + "mlp.down"))
                sd[p + "wout.weight"] = torch.cat(out, 1)
                continue
            if s.token_shift:
                sd[p + "shift"] = take(m + "shift")
            sd[p + "attention.wqkv.weight"] = torch.cat([take(m + "mix.q"), take(m + "mix.k"), take(m + "mix.v")])
            sd[p + "attention.wo.weight"] = take(m + "mix.o")
            if s.attention.distance_bias:
                sd[p + "attention.r1"], sd[p + "attention.r2"] = take(m + "mix.r1"), take(m + "mix.r2")
            if s.mlp is not None:
                sd[p + "ffn_norm.weight"] = take(m + "norm2")
                sd[p + "feed_forward.up.weight"], sd[p + "feed_forward.down.weight"] = take(m + "mlp.up"), take(m + "mlp.down")
                sd[p + "feed_forward.act"] = take(m + "mlp.act")
        extra = sorted(set(t) - used)
        if extra:
            raise KeyError(f"model.safetensors holds tensors this design does not have: {extra[:8]}")
        want = dict(self.named_parameters())
        for k, v in sd.items():
            if tuple(v.shape) != tuple(want[k].shape):
                raise ValueError(f"model.safetensors: {k} is {tuple(v.shape)}, config.json says {tuple(want[k].shape)}")
        return sd

    def tie_weights(self):
        """After loading: the head of a tied model is the embedding table itself."""
        if self.spec.tied_head:
            self.output.weight = self.tok_embeddings.weight

    # ------------------------------------------------------------------ setup
    def check_length(self, max_seq_length):
        if self.spec.max_positions and max_seq_length > self.spec.max_positions:
            raise ValueError(f"sequences of {max_seq_length} tokens: the model has {self.spec.max_positions} position vectors")

    def setup_caches(self, num_pages, page_size=128, spec=False, draft_num_pages=0, draft_budget=0, window_size=32,
                     max_positions=None, streaming=False, kv_dtype="bf16", kv_layout=None, decode_rows=None, slots=1,
                     state_ring=STATE_RING):
        """Per-layer pages and state rings for `slots` sequences.  kv_layout is ignored (there is one layout)."""
        if spec or streaming:
            raise NotImplementedError(f"{self.spec.design}: the compressed draft caches (SnapKV, StreamingLLM) select rows of "
                                      "per-head key / value pages, which this design does not keep")
        if kv_dtype != "bf16":
            raise NotImplementedError(f"{self.spec.design}: the fp8 cache is not available for this design")
        w = self.output.weight
        if w.dtype not in (torch.bfloat16, torch.float32):
            raise NotImplementedError("the layered decoder runs in bfloat16 or float32")
        dev, c = w.device, self.spec
        self.page_size, self.slots = page_size, slots
        self.state_ring = max(int(state_ring), 2)
        longest = max_positions or num_pages * page_size
        self._xspec, self._rings, self._act = [], [], []
        self._rotary, self._history = {}, None
        if c.bigram is not None:
            self._history = torch.zeros((num_pages, page_size), dtype=torch.int32, device=dev)
        for i, (layer, s) in enumerate(zip(self.layers, c.layers)):
            a = s.attention
            if s.parallel:
                r = a.rotary
                if r not in self._rotary:
                    yarn = (r.yarn.factor, r.yarn.original, r.yarn.fast, r.yarn.slow) if r.yarn else None
                    self._rotary[r] = ops.RotaryTable(r.dims, r.base, int(longest), yarn, device=dev)
                layer.attention.kv_cache = (LatentCache(num_pages, page_size, a.kv_rank, a.rot_dim, w.dtype).to(dev)
                                            if a.kv_from is None else self.layers[a.kv_from].attention.kv_cache)
                self._xspec.append(layer.attention.kernel_spec(c.norm_eps, self._rotary[r]))
                self._rings.append(None)
                self._act.append(None)
                continue
            layer.attention.kv_cache = SplitKVCache(num_pages, page_size, a.kv_heads, a.dim, a.vdim, w.dtype).to(dev)
            self._xspec.append(layer.attention.kernel_spec(c.norm_eps, longest))
            self._rings.append(torch.zeros((slots, self.state_ring, c.dim), dtype=torch.float32, device=dev)
                               if s.token_shift else None)
            self._act.append(layer.feed_forward.act.detach().float().contiguous() if s.mlp is not None else None)
        self.workspace = ops.AttnWorkspace(dev)
        self.decode_rows = tuple(sorted(set(int(r) for r in decode_rows))) if decode_rows else None
        self._pack_weights()
        self._ready = True

    def rollback_depth(self):
        """Tokens a sequence may be rolled back by (None: any number)."""
        return self.state_ring - 2 if any(r is not None for r in self._rings) else None

    def _streamed_weights(self):
        if self.output.weight.dtype != torch.bfloat16:
            return
        for i, b in enumerate(self.layers):
            if isinstance(b, ParallelLayer):
                yield b.attention.win.weight, False, "win", i
                yield b.attention.wuq.weight, False, "wuq", i
                if b.w13 is not None:
                    yield b.w13.weight, True, "gated", i
                yield b.wout.weight, False, "wout", i
                continue
            yield b.attention.wqkv.weight, False, "wqkv", i
            yield b.attention.wo.weight, False, "wo", i
            if b.feed_forward is not None:
                yield b.feed_forward.up.weight, False, "up", i
                yield b.feed_forward.down.weight, False, "down", i
        yield self.output.weight, False, "head", None

    def _decode_hows(self, role, N, K, int8, M, packed=True):
        if role in ("wo", "down", "wout"):
            return {self._project_how(M, N, K, packed)}
        if role == "gated":
            return {self._linear_how(M, N, K, True, int8, True if packed else None, "swiglu", False)}
        return {self._linear_how(M, N, K, False, int8, True if packed else None, "plain", False)}

    def _rowmajor_in_decode(self, w):
        # (a tied head is the embedding table: its rows are gathered in every step)
        return (self.spec.tied_head and w is self.output.weight) or super()._rowmajor_in_decode(w)

    # ------------------------------------------------------------------ the step
    def _linear(self, x2d, lin, **kw):
        if x2d.dtype == torch.float32:
            return F.linear(x2d, lin.weight)
        return super()._linear(x2d, lin, **kw)

    def _project_how(self, M, N, K, packed):
        """Where an output projection runs: a split-K GEMM up to its float32 planes ("skinny" | "tile" | "block"; the residual
        add + norm launch that follows is its combine), the skinny GEMM with 16-bit rows ("rows"), or the library."""
        how = choose(M, N, K, False, False, packed, "resid") if packed else "lib"
        if packed and how != "block" and (how == "fused" or use_split(M, N, K, "resid")):
            how = "tile"                     # the tile kernel's residual epilogue is 16-bit: take its K-split form instead
        if how in ("tile", "block", "skinny") and ops.linear_planes_count(how, M, N, K):
            return how
        return "rows" if how == "skinny" and ops.linear_supported(M, N, K) else "lib"

    def _project(self, inp, lin):
        """Output projection of a sub-layer, in a form ops.resid_norm adds to the residual."""
        pk = self._packed.get(id(lin.weight))
        M, K = inp.shape
        how = self._project_how(M, lin.weight.shape[0], K, pk is not None) if M <= 256 else "lib"
        if how in ops.PLANES_KINDS:
            return ops.linear_planes(inp, pk, how, self.workspace)
        if how == "rows":
            return ops.linear(inp, pk, workspace=self.workspace)
        self._last_M = M
        return F.linear(inp, self._resident(lin.weight))

    def _up_act(self, y, lin, act):
        """act(up . y): the activation is the GEMM's epilogue wherever a hand-written kernel runs it."""
        pk = self._packed.get(id(lin.weight))
        (M, K), N = y.shape, lin.weight.shape[0]
        how = self._linear_how(M, N, K, False, False, pk, "plain", False) if pk is not None and M <= 256 else "lib"
        if how == "fused":
            return ops.fused_linear(y, pk, xielu=act)
        if how == "block":
            return ops.linear_block(y, pk, workspace=self.workspace, xielu=act)
        if how == "skinny":
            return ops.linear(y, pk, workspace=self.workspace, xielu=act)
        self._last_M = M
        z = F.linear(y, self._resident(lin.weight))
        return ops.xielu(z, act, out=z)

    def _gated(self, y, lin, out):
        """gelu(gate . y) * (up . y) into `out`: the GEMM's epilogue wherever a hand-written kernel runs it."""
        pk = self._packed.get(id(lin.weight))
        (M, K), N = y.shape, lin.weight.shape[0]
        how = self._linear_how(M, N, K, True, False, pk, "swiglu", False) if pk is not None and M <= 256 else "lib"
        if out.stride(0) % 8 or out.data_ptr() % 16:
            how = "lib"
        if how == "fused":
            return ops.fused_linear(y, pk, swiglu=True, gelu=True, out=out)
        if how == "block":
            return ops.linear_block(y, pk, swiglu=True, gelu=True, workspace=self.workspace, out=out)
        if how == "skinny":
            return ops.linear(y, pk, swiglu=True, gelu=True, workspace=self.workspace, out=out)
        self._last_M = M
        z = F.linear(y, self._resident(lin.weight))
        return ops.gelu_mul(z[:, :N // 2], z[:, N // 2:], out=out)

    def _parallel(self, i, layer, y, rows, tab: PageTable, ctx):
        """mixer(y) + feed_forward(y) in a form ops.resid_norm adds to the residual."""
        att, s = layer.attention, self._xspec[i]
        cache = att.kv_cache.rows
        z = self._linear(y, att.win)
        cq = ops.latent_append(z, s, cache, rows, tab.indices, tab.indptr, tab.max_pages)
        q = self._linear(cq, att.wuq)
        side = torch.empty((y.shape[0], layer.wout.weight.shape[1]), dtype=y.dtype, device=y.device)
        heads = side[:, :layer.heads_out].unflatten(1, (s.H, s.vdim))
        ops.latent_attention(q, s, cache, rows, tab.indices, tab.indptr, tab.max_pages, self.workspace, heads,
                             gate=z[:, z.shape[1] - s.H:] if att.spec.gate else None, ctx=ctx)
        if layer.w13 is not None:
            self._gated(y, layer.w13, side[:, layer.heads_out:])
        return self._project(side, layer.wout)

    def _embed(self, flat, rows, tab: PageTable):
        c = self.spec
        if c.bigram is not None:
            return ops.embed_bigram(flat, self.tok_embeddings.weight, self.pair_embeddings.weight, self.embed_norm.weight, c.norm_eps,
                                    c.bigram.mul_before, c.bigram.mul_token, self._history, rows, tab.indices, tab.indptr)
        return ops.embed_pos(flat, self.tok_embeddings.weight,
                             self.pos_embeddings.weight if self.pos_embeddings is not None else None, rows, c.embed_scale)

    def _step(self, idx, offsets, qo_indptr, tab: PageTable, n_max=None, head_rows=None):
        """One step over `idx` ([B, n], or flat with n_max): embed -> layers -> norm -> head -> argmax.  head_rows: the flat
        rows whose logits are wanted (None: all)."""
        assert self._ready, "call setup_caches first"
        c = self.spec
        flat = idx.reshape(-1).contiguous()
        rows = ops.StepRows(qo_indptr, offsets, idx.shape[1] if idx.dim() == 2 else n_max, tab.slots)
        x = self._embed(flat, rows, tab)
        ctx = None
        if tab.lengths is not None and self.output.weight.dtype == torch.bfloat16:
            ctx = ops.LatentContext(*tab.lengths, x.device)
        delta = None
        for i, layer in enumerate(self.layers):
            att, kvc = layer.attention, layer.attention.kv_cache
            x, y = ops.resid_norm(x, delta, layer.attention_norm.weight, c.norm_eps,
                                  shift=getattr(layer, "shift", None), ring=self._rings[i], rows=rows)
            if isinstance(layer, ParallelLayer):
                delta = self._parallel(i, layer, y, rows, tab, ctx)
                if self._layer_hook is not None:
                    self._layer_hook(i, x, delta)
                continue
            qkv = self._linear(y, att.wqkv)
            o = ops.extended_attention(qkv, self._xspec[i], kvc.k_cache, kvc.v_cache, rows, tab.indices, tab.indptr,
                                       tab.max_pages, self.workspace)
            delta = self._project(o, att.wo)
            if layer.feed_forward is not None:
                x, y = ops.resid_norm(x, delta, layer.ffn_norm.weight, c.norm_eps)
                delta = self._project(self._up_act(y, layer.feed_forward.up, self._act[i]), layer.feed_forward.down)
            if self._layer_hook is not None:
                self._layer_hook(i, x, delta)
        if self.skip_head:
            return None
        x, y = ops.resid_norm(x, delta, self.norm.weight, c.norm_eps, out_scale=c.logit_scale)
        if head_rows is not None:
            y = y.index_select(0, head_rows)
        logits = self._linear(y, self.output)
        if c.logit_softcap is not None:
            logits = ops.softcap_(logits, c.logit_softcap)
        self._last_logits = logits
        tokens = self._argmax(logits)
        return tokens.view(idx.shape) if head_rows is None else tokens

    _layer_hook = None       # called as (layer index, residual, pending delta): diagnostics

    def forward(self, idx, input_pos, kv_append_indptr, tab: PageTable, n_max=None, head_rows=None):
        return self._step(idx, input_pos, kv_append_indptr, tab, n_max, head_rows)

    def prefill(self, idx, input_pos, kv_append_indptr, tab: PageTable, is_last=False, draft_tab=None, ctx_len=None,
                n_max=None, head_rows=None):
        return self._step(idx, input_pos, kv_append_indptr, tab, n_max, head_rows)

    def verify(self, *a, **k):
        raise NotImplementedError(f"{self.spec.design}: no self-speculation cache")

    draft_forward = stream_prefill = verify
