"""Tensor-level wrappers over the C ABI (include/magicdec_hip.h).

These are the seven ``mylib::*`` operators of the reference (Engine/utils.py:31-66,
Engine/SnapKV/backend.py:56-107, Engine/SnapKV/model.py:133-156) plus the fused
small ops of the decode loop, with the same tensor-level signatures, backed by
hand-written gfx950 kernels.  Differences from the reference's op boundary:

* no hidden ``plan()`` state: the page table is passed to the attention op
  explicitly and read on the device (no host sync, graph-capturable);
* tensors must live on the GPU; there is no CPU implementation here
  (``MagicDecHipError`` if the library is missing, ``ValueError`` for CPU tensors).
"""
from __future__ import annotations

import ctypes
import math

import torch

from . import _lib
from ._lib import MagicDecHipError, check  # noqa: F401

PAGE_SIZE = 128
MD_KV_BF16, MD_KV_FP8_E4M3 = 0, 1      # include/magicdec_hip.h
MD_KV_LAYOUT_HND = 0x100
FP8_DTYPE = torch.float8_e4m3fn
KV_LAYOUTS = ("NHD", "HND")


def _kv_geom(kv_cache, kv_layout):
    """(page_size, KH, D) of a paged cache [pages, 2, page_size, KH, D] ("NHD", the reference's layout:
    Engine/SnapKV/backend.py:30) or [pages, 2, KH, page_size, D] ("HND", rows of a kv head contiguous)."""
    if kv_layout not in KV_LAYOUTS:
        raise ValueError(f"kv_layout must be one of {KV_LAYOUTS}, got {kv_layout!r}")
    if kv_cache.dim() != 5 or kv_cache.shape[1] != 2 or not kv_cache.is_contiguous():
        raise ValueError("paged KV cache must be a contiguous [pages, 2, ., ., D] tensor")
    if kv_layout == "HND":
        return kv_cache.shape[3], kv_cache.shape[2], kv_cache.shape[4]
    return kv_cache.shape[2], kv_cache.shape[3], kv_cache.shape[4]


def _kv_args(kv_cache, kv_scales, kv_layout="NHD"):
    """(kv_dtype | layout flag, k_scale ptr, v_scale ptr) for a paged cache: bf16 caches take no scales, e4m3fn
    caches need per-kv-head float32 dequantisation scales `(k_scale[KH], v_scale[KH])`."""
    flag = MD_KV_LAYOUT_HND if kv_layout == "HND" else 0
    if kv_cache.dtype == torch.bfloat16:
        return MD_KV_BF16 | flag, None, None
    if kv_cache.dtype != FP8_DTYPE:
        raise TypeError(f"paged KV cache must be bfloat16 or float8_e4m3fn, got {kv_cache.dtype}")
    if kv_scales is None:
        raise ValueError("an fp8 KV cache needs kv_scales=(k_scale, v_scale)")
    ks, vs = kv_scales
    KH = _kv_geom(kv_cache, kv_layout)[1]
    for t in (ks, vs):
        if t.dtype != torch.float32 or t.numel() != KH or not t.is_contiguous() or not t.is_cuda:
            raise ValueError("kv scales must be contiguous float32 [KH] tensors on the GPU")
    return MD_KV_FP8_E4M3 | flag, _p(ks), _p(vs)


def _p(t):
    return ctypes.c_void_p(t.data_ptr()) if t is not None else None


def _stream():
    return ctypes.c_void_p(torch.cuda.current_stream().cuda_stream)


def _gpu(*ts):
    for t in ts:
        if t is not None and not t.is_cuda:
            raise ValueError("magicdec_amd.ops: tensors must be on the GPU (no CPU path exists)")


def _i32(t):
    if t.dtype != torch.int32:
        raise TypeError("page-table tensors must be int32")
    return t


def _row_stride(t):
    """[rows, heads, D] view whose last two dims are dense; returns the row stride in elements."""
    if t.dim() != 3 or t.stride(2) != 1 or t.stride(1) != t.shape[2]:
        raise ValueError("expected a [rows, heads, D] tensor with dense (heads, D)")
    return t.stride(0)


# ----------------------------------------------------------------------------- K4
def update_kv(k, v, kv_append_indptr, kv_cache, kv_page_indices, kv_page_indptr, kv_page_lastlen, n_max=None,
              kv_scales=None, kv_layout="NHD"):
    """mylib::update_kv (Engine/utils.py:31-54).  In place on kv_cache."""
    _gpu(k, v, kv_cache)
    B = kv_page_indptr.numel() - 1
    page_size, KH, D = _kv_geom(kv_cache, kv_layout)
    if n_max is None:
        n_max = (k.shape[0] + B - 1) // B if B > 0 else 0
        n_max = max(n_max, 1)
    lib = _lib.load()
    check(lib.md_append_paged_kv(_p(k), _p(v), _row_stride(k), _row_stride(v), _p(_i32(kv_append_indptr)),
                                 _p(kv_cache), _p(_i32(kv_page_indices)), _p(_i32(kv_page_indptr)),
                                 _p(_i32(kv_page_lastlen)), B, n_max, KH, D, page_size,
                                 *_kv_args(kv_cache, kv_scales, kv_layout), _stream()),
          "md_append_paged_kv")


def page_overflow_count(reset=True):
    """KV rows dropped by the append kernels because their request's last page was full (see
    md_page_overflow_count).  Synchronises with the device: call it per batch, not per step."""
    n = ctypes.c_uint(0)
    check(_lib.load().md_page_overflow_count(ctypes.byref(n), 1 if reset else 0), "md_page_overflow_count")
    return int(n.value)


# ----------------------------------------------------------------------------- K5
class RopeTable:
    """Host-precomputed cos/sin table on the device (float32 [max_pos, D/2, 2])."""

    def __init__(self, max_pos, head_dim, rope_theta, rope_scale, low_freq_factor=None, high_freq_factor=None,
                 old_context_len=None, device="cuda"):
        lib = _lib.load()
        host = torch.empty(max_pos, head_dim // 2, 2, dtype=torch.float32)
        llama31 = low_freq_factor is not None and high_freq_factor is not None
        check(lib.md_rope_fill_table_host(ctypes.c_void_p(host.data_ptr()), max_pos, head_dim, float(rope_theta),
                                          float(rope_scale), float(low_freq_factor) if llama31 else 0.0,
                                          float(high_freq_factor) if llama31 else 0.0,
                                          float(old_context_len) if llama31 else 0.0),
              "md_rope_fill_table_host")
        self.table = host.to(device)
        self.max_pos = max_pos
        self.head_dim = head_dim


def rope(q, k, indptr, offsets, table: RopeTable, n_max=None):
    """mylib::rope / mylib::draft_rope (Engine/SnapKV/model.py:133-156): returns new (q, k)."""
    _gpu(q, k)
    B = indptr.numel() - 1
    H, D = q.shape[1], q.shape[2]
    KH = k.shape[1] if k is not None else 0
    if n_max is None:
        n_max = max((q.shape[0] + B - 1) // B, 1)
    q_out = torch.empty((q.shape[0], H, D), dtype=q.dtype, device=q.device)
    k_out = torch.empty((k.shape[0], KH, D), dtype=k.dtype, device=k.device) if k is not None else None
    lib = _lib.load()
    check(lib.md_rope(_p(q), _p(k), _row_stride(q), _row_stride(k) if k is not None else 0, _p(q_out), _p(k_out),
                      _p(_i32(indptr)), _p(_i32(offsets)), B, n_max, H, KH, D, _p(table.table), table.max_pos,
                      _stream()), "md_rope")
    return q_out, k_out


def rope_append(q, k, v, indptr, offsets, table: RopeTable, kv_cache, page_indices, page_indptr, last_page_len,
                kv_cache2=None, page_indices2=None, page_indptr2=None, last_page_len2=None, n_max=None,
                kv_scales=None, kv_layout="NHD"):
    """Fused mylib::rope + mylib::update_kv (+ second cache for self-spec verify).  Returns rotated q.
    kv_cache may be fp8 (with kv_scales) and/or HND (kv_layout); kv_cache2 is always bf16 NHD."""
    _gpu(q, k, v, kv_cache, kv_cache2)
    B = indptr.numel() - 1
    H, D = q.shape[1], q.shape[2]
    KH = k.shape[1]
    if n_max is None:
        n_max = max((q.shape[0] + B - 1) // B, 1)
    q_out = torch.empty((q.shape[0], H, D), dtype=q.dtype, device=q.device)
    lib = _lib.load()
    check(lib.md_rope_append(_p(q), _p(k), _p(v), _row_stride(q), _row_stride(k), _row_stride(v), _p(q_out),
                             _p(_i32(indptr)), _p(_i32(offsets)), B, n_max, H, KH, D, _p(table.table), table.max_pos,
                             _p(kv_cache), _p(_i32(page_indices)), _p(_i32(page_indptr)), _p(_i32(last_page_len)),
                             _p(kv_cache2), _p(page_indices2), _p(page_indptr2), _p(last_page_len2),
                             _kv_geom(kv_cache, kv_layout)[0], *_kv_args(kv_cache, kv_scales, kv_layout), _stream()),
          "md_rope_append")
    return q_out


# ----------------------------------------------------------------------------- K1/K2/K3
class AttnWorkspace:
    """Scratch for split-KV partials, grown on demand (never inside a captured graph)."""

    def __init__(self, device="cuda"):
        self.device = device
        self.buf = torch.empty(1 << 20, dtype=torch.uint8, device=device)
        self._retired = []     # outgrown buffers stay allocated: captured hipGraphs have their addresses baked in

    def get(self, nbytes):
        if self.buf.numel() < nbytes:
            self._retired.append(self.buf)
            self.buf = torch.empty(int(nbytes * 1.25) + 256, dtype=torch.uint8, device=self.device)
        return self.buf


def paged_attention(q, kv_cache, qo_indptr, page_indices, page_indptr, last_page_len, n_max, max_pages_per_req,
                    workspace: AttnWorkspace, causal=True, sm_scale=None, out=None, kv_scales=None,
                    kv_layout="NHD"):
    """mylib::target_decode / target_prefill / draft_decode / draft_prefill
    (Engine/SnapKV/backend.py:56-107): flashinfer BatchPrefillWithPagedKVCacheWrapper.run with the
    plan() arguments passed explicitly."""
    _gpu(q, kv_cache)
    B = page_indptr.numel() - 1
    H, D = q.shape[1], q.shape[2]
    page_size, KH, _ = _kv_geom(kv_cache, kv_layout)
    if sm_scale is None:
        sm_scale = 1.0 / math.sqrt(D)
    if out is None:
        out = torch.empty((q.shape[0], H, D), dtype=q.dtype, device=q.device)
    lib = _lib.load()
    nbytes = lib.md_paged_attn_workspace_bytes(B, n_max, H, KH, D, max_pages_per_req, page_size)
    ws = workspace.get(nbytes)
    check(lib.md_paged_attn(_p(q), _row_stride(q), _p(kv_cache), _p(out), _p(_i32(qo_indptr)), _p(_i32(page_indices)),
                            _p(_i32(page_indptr)), _p(_i32(last_page_len)), B, n_max, H, KH, D, page_size,
                            1 if causal else 0, float(sm_scale), max_pages_per_req,
                            *_kv_args(kv_cache, kv_scales, kv_layout),
                            _p(ws), ws.numel(), _stream()),
          "md_paged_attn")
    return out


# ----------------------------------------------------------------------------- K6
def snapkv_select(q_win, kv_cache, page_indices, page_indptr, ctx_len, window, budget, pool_kernel, draft_cache,
                  draft_page_indices, draft_page_indptr, draft_last_page_len, workspace: AttnWorkspace,
                  return_scores=False, kv_scales=None, kv_layout="NHD"):
    """Attention.gen_draft_kv (Engine/SnapKV/model.py:389-439): writes budget rows per request and kv head
    into draft_cache; returns the selected positions [B, KH, budget-window] int32 (reference order).
    kv_layout describes kv_cache (the source); draft_cache is always bf16 NHD."""
    _gpu(q_win, kv_cache, draft_cache)
    B = page_indptr.numel() - 1
    H, D = q_win.shape[1], q_win.shape[2]
    page_size, KH, _ = _kv_geom(kv_cache, kv_layout)
    if not q_win.is_contiguous():
        q_win = q_win.contiguous()
    idx = torch.empty((B, KH, budget - window), dtype=torch.int32, device=q_win.device)
    lib = _lib.load()
    nbytes = lib.md_snapkv_workspace_bytes(B, H, KH, ctx_len, window)
    if nbytes == 0:
        raise ValueError("md_snapkv_workspace_bytes: bad shape")
    ws = workspace.get(nbytes + 512)
    off = (-ws.data_ptr()) % 256
    check(lib.md_snapkv_select(_p(q_win), _p(kv_cache), _p(_i32(page_indices)), _p(_i32(page_indptr)), B, H, KH, D,
                               page_size, ctx_len, window, budget, pool_kernel, _p(draft_cache),
                               _p(_i32(draft_page_indices)), _p(_i32(draft_page_indptr)), _p(_i32(draft_last_page_len)),
                               _p(idx), *_kv_args(kv_cache, kv_scales, kv_layout), ctypes.c_void_p(ws.data_ptr() + off),
                               nbytes, _stream()), "md_snapkv_select")
    if return_scores:
        soff = lib.md_snapkv_scores_offset(B, H, KH, ctx_len, window)
        n = B * KH * (ctx_len - window)
        sc = ws[off + soff: off + soff + 2 * n].view(torch.bfloat16).view(B, KH, ctx_len - window).clone()
        return idx, sc
    return idx


# ----------------------------------------------------------------------------- K7
def streaming_shift_append(k_new, v_new, kv_cache, n_new, kv_len, sink, pages_per_req):
    """In-place equivalent of KVCache.prefill's eviction branch (Engine/StreamingLLM/model_draft.py:122-134)."""
    _gpu(k_new, v_new, kv_cache)
    B = k_new.shape[0] // n_new
    KH, D = kv_cache.shape[3], kv_cache.shape[4]
    lib = _lib.load()
    check(lib.md_streaming_shift_append(_p(k_new), _p(v_new), _row_stride(k_new), _row_stride(v_new), _p(kv_cache), B,
                                        n_new, kv_len, sink, pages_per_req, KH, D, kv_cache.shape[2], _stream()),
          "md_streaming_shift_append")


def streaming_rotate(kv_cache, rot_cache, B, valid_len, pages_per_req, table: RopeTable):
    """Rotated clone of the draft cache (Engine/StreamingLLM/model_draft.py:112-118,135-143): K rotated by
    slot position, V copied, rows [0, valid_len) of every request.  rot_cache may be kv_cache (in place)."""
    _gpu(kv_cache, rot_cache)
    KH, D = kv_cache.shape[3], kv_cache.shape[4]
    lib = _lib.load()
    check(lib.md_streaming_rotate(_p(kv_cache), _p(rot_cache), B, valid_len, pages_per_req, KH, D, kv_cache.shape[2],
                                  _p(table.table), table.max_pos, _stream()), "md_streaming_rotate")


# ----------------------------------------------------------------------------- K8
MD_W_BF16, MD_W_INT8 = 0, 1
EPI_NONE, EPI_SWIGLU, EPI_GEGLU = 0, 1, 3


def linear_supported(M, N, K, swiglu=False):
    """True when md_linear (the weight-streaming skinny GEMM) takes this shape; otherwise use a library GEMM."""
    return bool(_lib.load().md_linear_supported(int(M), int(N), int(K), EPI_SWIGLU if swiglu else EPI_NONE))


class PackedWeight:
    """A linear's weight in the streaming layout of md_linear (include/magicdec_hip.h: w_packed = 1):
    [ceil(N/32)][K/16][64 lanes][8] -- element (t, s, lane, e) = W[32t + lane%32][16s + 8*(lane/32) + e], rows past N
    zero; for swiglu=True tile t = rows 16t..16t+15 of w1 then rows 16t..16t+15 of w3 (weight = [w1; w3], N = 2I).
    Built once at load time (a torch permute: plumbing); bf16 or int8."""

    def __init__(self, weight, swiglu=False):
        N, K = weight.shape
        if K % 16:
            raise ValueError("PackedWeight needs K % 16 == 0")
        self.N, self.K, self.swiglu, self.dtype = N, K, swiglu, weight.dtype
        if swiglu:
            inter = N // 2
            t = (inter + 15) // 16
            w1 = torch.zeros((t * 16, K), dtype=weight.dtype, device=weight.device)
            w3 = torch.zeros((t * 16, K), dtype=weight.dtype, device=weight.device)
            w1[:inter], w3[:inter] = weight[:inter], weight[inter:]
            rows = torch.cat([w1.view(t, 16, K), w3.view(t, 16, K)], dim=1)          # [t, 32, K]
        else:
            t = (N + 31) // 32
            rows = torch.zeros((t * 32, K), dtype=weight.dtype, device=weight.device)
            rows[:N] = weight
            rows = rows.view(t, 32, K)
        # [t, j, s, kh, e] -> [t, s, kh, j, e]
        self.data = rows.view(t, 32, K // 16, 2, 8).permute(0, 2, 3, 1, 4).contiguous()

    def unpack(self):
        """The row-major [N, K] tensor this copy was built from (the inverse permute: plumbing).  Used to re-materialise
        a row-major weight that was released after prefill (Transformer.release_rowmajor): the streaming layout is then
        the ONE resident copy of the weight."""
        t, K = self.data.shape[0], self.K
        rows = self.data.permute(0, 3, 1, 2, 4).reshape(t, 32, K)      # [t, s, kh, j, e] -> [t, j, (s, kh, e)]
        if not self.swiglu:
            return rows.view(t * 32, K)[:self.N] if t * 32 != self.N else rows.view(t * 32, K)
        inter = self.N // 2
        out = torch.empty((self.N, K), dtype=self.data.dtype, device=self.data.device)
        out[:inter].copy_(rows[:, :16].reshape(t * 16, K)[:inter])
        out[inter:].copy_(rows[:, 16:].reshape(t * 16, K)[:inter])
        return out


def _act_numbers(act):
    if act.dtype != torch.float32 or act.numel() != 2 or not act.is_cuda or not act.is_contiguous():
        raise ValueError("xielu: float32 act[2] on the GPU expected")
    return _p(act)


def linear(x, weight, bias=None, scales=None, swiglu=False, workspace: "AttnWorkspace" = None, out=None,
           pro: "DeferredNorm" = None, xielu=None, gelu=False):
    """F.linear(x, weight, bias) for M = x.shape[0] <= 256 rows on the hand-written gfx950 skinny GEMM (md_linear).
    x [M, K] bf16 with unit inner stride (row stride free); weight: a contiguous [N, K] tensor or a PackedWeight
    (streaming layout), bf16 -- or int8 with bf16 per-row `scales` (WeightOnlyInt8Linear semantics:
    bf16(x.w^T) * scales).  swiglu=True: weight = [w1; w3] (N = 2*I rows) and the result is
    silu(x.w1^T) * (x.w3^T) [M, I] with the reference's bf16 rounding points.
    pro (bf16 weights): x is pro.h, the un-normalised hidden state, and is normalised on the fly (md_linear_normed).
    xielu (bf16 weights): the two numbers of the activation applied to the result (md_linear_xielu).
    gelu (with swiglu): gelu_tanh(h1) * h3 instead, fp32 up to the one rounding of the product."""
    packed = isinstance(weight, PackedWeight)
    wt = weight.data if packed else weight
    _gpu(x, wt, bias, scales)
    if x.dim() != 2 or x.stride(1) != 1:
        raise ValueError("linear expects x [M, K] with unit inner stride")
    M, K = x.shape
    if packed:
        if weight.swiglu != swiglu:
            raise ValueError("PackedWeight was packed for a different epilogue")
        N, wk = weight.N, weight.K
    else:
        if weight.dim() != 2 or not weight.is_contiguous():
            raise ValueError("linear expects a contiguous weight [N, K]")
        N, wk = weight.shape
    if wk != K:
        raise ValueError(f"linear: x has K={K}, weight has K={wk}")
    if wt.dtype == torch.int8:
        if scales is None:
            raise ValueError("int8 weights need per-row scales")
        wd = MD_W_INT8
    elif wt.dtype == torch.bfloat16:
        wd = MD_W_BF16
    else:
        raise TypeError(f"linear: weight dtype {wt.dtype} unsupported (bf16 or int8)")
    epi = (EPI_GEGLU if gelu else EPI_SWIGLU) if swiglu else EPI_NONE
    n_out = N // 2 if swiglu else N
    if out is None:
        out = torch.empty((M, n_out), dtype=x.dtype, device=x.device)
    lib = _lib.load()
    nbytes = lib.md_linear_workspace_bytes(M, N, K, epi)
    ws = None
    if nbytes:
        if workspace is None:
            raise ValueError("linear: this shape splits K and needs a workspace")
        ws = workspace.get(nbytes + 256)
        off = (-ws.data_ptr()) % 256
    wsp = ctypes.c_void_p(ws.data_ptr() + off) if ws is not None else None
    if xielu is not None:
        if wd != MD_W_BF16 or swiglu or pro is not None or bias is not None:
            raise ValueError("linear: the xIELU epilogue takes bf16 weights and nothing beside it")
        check(lib.md_linear_xielu(_p(x), x.stride(0), _p(wt), 1 if packed else 0, _act_numbers(xielu), _p(out), out.stride(0),
                                  M, N, K, wsp, nbytes, _stream()), "md_linear_xielu")
        return out
    if pro is not None:
        if wd != MD_W_BF16:
            raise TypeError("linear: the deferred norm needs bf16 weights")
        a = _lib.FusedLinearArgs()             # _set_pro's checks (x is pro.h, ssq [M, K / 32] fp32, bf16 weight [K])
        _set_pro(a, x, pro)
        check(lib.md_linear_normed(_p(x), x.stride(0), _p(pro.ssq), pro.ssq.shape[1], _p(pro.weight), pro.eps, _p(wt),
                                   1 if packed else 0, _p(bias), _p(out), out.stride(0), M, N, K, epi, wsp, nbytes,
                                   _stream()),
              "md_linear_normed")
        return out
    check(lib.md_linear(_p(x), x.stride(0), _p(wt), wd, 1 if packed else 0, _p(scales), _p(bias), _p(out),
                        out.stride(0), M, N, K, epi, wsp, nbytes, _stream()),
          "md_linear")
    return out


def linear_add_rmsnorm_supported(M, N, K):
    """True when md_linear_add_rmsnorm takes this shape (an md_linear shape whose K is split, N <= 8192)."""
    return bool(_lib.load().md_linear_add_rmsnorm_supported(int(M), int(N), int(K)))


def linear_add_rmsnorm(x, weight, resid, norm_weight, eps, bias=None, scales=None, workspace: "AttnWorkspace" = None):
    """(h, y) = (resid + F.linear(x, W, bias), rmsnorm(h) * norm_weight) on md_linear with the residual add and the norm
    fused into its split-K combine launch -- bit-identical to linear() followed by add_rmsnorm()."""
    packed = isinstance(weight, PackedWeight)
    wt = weight.data if packed else weight
    _gpu(x, wt, bias, scales, resid, norm_weight)
    if x.dim() != 2 or x.stride(1) != 1 or resid.dim() != 2 or resid.stride(1) != 1:
        raise ValueError("linear_add_rmsnorm expects 2-D x / resid with unit inner stride")
    M, K = x.shape
    N = weight.N if packed else weight.shape[0]
    if packed and weight.swiglu:
        raise ValueError("linear_add_rmsnorm: the weight was packed for the SwiGLU epilogue")
    if resid.shape != (M, N) or norm_weight.numel() != N:
        raise ValueError("linear_add_rmsnorm: resid must be [M, N], norm_weight [N]")
    wd = MD_W_INT8 if wt.dtype == torch.int8 else MD_W_BF16
    if wd == MD_W_INT8 and scales is None:
        raise ValueError("int8 weights need per-row scales")
    lib = _lib.load()
    nbytes = lib.md_linear_workspace_bytes(M, N, K, EPI_NONE)
    if workspace is None or not nbytes:
        raise ValueError("linear_add_rmsnorm: needs a workspace and a shape whose K is split")
    ws = workspace.get(nbytes + 256)
    off = (-ws.data_ptr()) % 256
    h = torch.empty((M, N), dtype=x.dtype, device=x.device)
    y = torch.empty((M, N), dtype=x.dtype, device=x.device)
    check(lib.md_linear_add_rmsnorm(_p(x), x.stride(0), _p(wt), wd, 1 if packed else 0, _p(scales), _p(bias), _p(resid),
                                    resid.stride(0), _p(norm_weight), float(eps), _p(h), _p(y), M, N, K,
                                    ctypes.c_void_p(ws.data_ptr() + off), nbytes, _stream()), "md_linear_add_rmsnorm")
    return h, y


# ----------------------------------------------------------------------------- K8b, K split over workgroups
def fused_split_supported(M, N, K):
    """md_linear_fused_split takes this shape (M <= 256, K % 128 == 0, N % 32 == 0)."""
    return 1 <= M <= 256 and K >= 128 and K % 128 == 0 and N >= 32 and N % 32 == 0


def _split_ws(lib, M, N, K, workspace):
    nbytes = lib.md_linear_fused_split_workspace_bytes(M, N, K)
    if not nbytes or workspace is None:
        raise ValueError("fused_split_linear: needs a workspace and a supported shape")
    ws = workspace.get(nbytes + 256)
    return ctypes.c_void_p(ws.data_ptr() + (-ws.data_ptr()) % 256), nbytes


def fused_split_linear(x, weight: "PackedWeight", bias=None, workspace: "AttnWorkspace" = None):
    """F.linear(x, W, bias) on the tile kernel with K also split over workgroups + the fixed-order combine launch
    (md_linear_fused_split; csrc/tilegemm.hip)."""
    _gpu(x, weight.data, bias)
    if x.dim() != 2 or x.stride(1) != 1 or weight.swiglu:
        raise ValueError("fused_split_linear expects a 2-D x with unit inner stride and a plain packed weight")
    M, K = x.shape
    N = weight.N
    lib = _lib.load()
    wsp, nbytes = _split_ws(lib, M, N, K, workspace)
    out = torch.empty((M, N), dtype=x.dtype, device=x.device)
    check(lib.md_linear_fused_split(_p(x), x.stride(0), _p(weight.data), _p(bias), _p(out), out.stride(0), M, N, K, wsp,
                                    nbytes, _stream()), "md_linear_fused_split")
    return out


def fused_split_linear_add_rmsnorm(x, weight: "PackedWeight", resid, norm_weight, eps, bias=None,
                                   workspace: "AttnWorkspace" = None):
    """(h, y) = (resid + F.linear(x, W, bias), rmsnorm(h) * norm_weight): the split tile kernel + ONE combine launch that
    adds the slices in order, the residual, and normalises (md_linear_fused_split_add_rmsnorm) -- bit-identical to
    fused_split_linear() followed by add_rmsnorm()."""
    _gpu(x, weight.data, bias, resid, norm_weight)
    if x.dim() != 2 or x.stride(1) != 1 or resid.dim() != 2 or resid.stride(1) != 1 or weight.swiglu:
        raise ValueError("fused_split_linear_add_rmsnorm expects 2-D x / resid with unit inner stride and a plain packed weight")
    M, K = x.shape
    N = weight.N
    if resid.shape != (M, N) or norm_weight.numel() != N:
        raise ValueError("fused_split_linear_add_rmsnorm: resid must be [M, N], norm_weight [N]")
    lib = _lib.load()
    wsp, nbytes = _split_ws(lib, M, N, K, workspace)
    h = torch.empty((M, N), dtype=x.dtype, device=x.device)
    y = torch.empty((M, N), dtype=x.dtype, device=x.device)
    check(lib.md_linear_fused_split_add_rmsnorm(_p(x), x.stride(0), _p(weight.data), _p(bias), _p(resid), resid.stride(0),
                                                _p(norm_weight), float(eps), _p(h), _p(y), M, N, K, wsp, nbytes, _stream()),
          "md_linear_fused_split_add_rmsnorm")
    return h, y


# ----------------------------------------------------------------------------- K8c
def linear_block_supported(M, N, K, swiglu=False):
    """True when md_linear_block (csrc/blockgemm.hip: the block-tile GEMM of the 129..256-row verify linears) takes
    this shape (M <= 256, N % 128 == 0, K % 64 == 0)."""
    return bool(_lib.load().md_linear_block_supported(int(M), int(N), int(K), EPI_SWIGLU if swiglu else EPI_NONE))


def _block_ws(lib, M, N, K, force, workspace):
    nbytes = lib.md_linear_block_workspace_bytes(M, N, K, 1 if force else 0)
    if not nbytes:
        return None, 0
    if workspace is None:
        raise ValueError("linear_block: this shape splits K and needs a workspace")
    ws = workspace.get(nbytes + 256)
    return ctypes.c_void_p(ws.data_ptr() + (-ws.data_ptr()) % 256), nbytes


def _block_args(x, weight, swiglu):
    if not isinstance(weight, PackedWeight) or weight.dtype != torch.bfloat16:
        raise TypeError("linear_block streams a bf16 PackedWeight")
    _gpu(x, weight.data)
    if x.dim() != 2 or x.stride(1) != 1 or x.dtype != torch.bfloat16:
        raise ValueError("linear_block expects x [M, K] bf16 with unit inner stride")
    if weight.K != x.shape[1]:
        raise ValueError(f"linear_block: x has K={x.shape[1]}, weight has K={weight.K}")
    if weight.swiglu != swiglu:
        raise ValueError("PackedWeight was packed for a different epilogue")
    return x.shape[0], weight.N, weight.K


def _block_bias(bias, N):
    """md_linear_block reads the bias as 16-byte vectors of N bf16 values."""
    if bias is None:
        return
    _gpu(bias)
    if bias.dtype != torch.bfloat16 or bias.numel() != N or not bias.is_contiguous() or bias.data_ptr() % 16:
        raise ValueError(f"linear_block: bias must be a contiguous, 16-byte aligned bf16 vector of {N} elements")


def linear_block(x, weight: "PackedWeight", bias=None, swiglu=False, workspace: "AttnWorkspace" = None, out=None,
                 xielu=None, gelu=False):
    """F.linear(x, W, bias) (or silu(x.w1^T) * (x.w3^T) for swiglu=True, weight = [w1; w3]) for 129..256 rows on the
    block-tile GEMM md_linear_block; same contract and rounding points as linear()."""
    M, N, K = _block_args(x, weight, swiglu)
    _block_bias(bias, N)
    n_out = N // 2 if swiglu else N
    if out is None:
        out = torch.empty((M, n_out), dtype=x.dtype, device=x.device)
    else:
        _gpu(out)
        if out.dtype != torch.bfloat16 or out.dim() != 2 or out.shape != (M, n_out) or out.stride(1) != 1:
            raise ValueError("linear_block: out must be bf16 [M, N_out] with unit inner stride")
    lib = _lib.load()
    wsp, nbytes = _block_ws(lib, M, N, K, False, workspace)
    if xielu is not None:
        if swiglu or bias is not None:
            raise ValueError("linear_block: the xIELU epilogue takes nothing beside it")
        check(lib.md_linear_block_xielu(_p(x), x.stride(0), _p(weight.data), _act_numbers(xielu), _p(out), out.stride(0), M, N,
                                        K, wsp, nbytes, _stream()), "md_linear_block_xielu")
        return out
    check(lib.md_linear_block(_p(x), x.stride(0), _p(weight.data), _p(bias), _p(out), out.stride(0), M, N, K,
                              (EPI_GEGLU if gelu else EPI_SWIGLU) if swiglu else EPI_NONE, wsp, nbytes, _stream()),
          "md_linear_block")
    return out


def linear_block_add_rmsnorm(x, weight: "PackedWeight", resid, norm_weight, eps, bias=None,
                             workspace: "AttnWorkspace" = None):
    """(h, y) = (resid + F.linear(x, W, bias), rmsnorm(h) * norm_weight): md_linear_block with the residual add and the
    norm in its combine launch -- the combine kernel of linear_add_rmsnorm (same rounding points)."""
    M, N, K = _block_args(x, weight, False)
    _block_bias(bias, N)
    _gpu(resid, norm_weight)
    if resid.dim() != 2 or resid.stride(1) != 1 or resid.shape != (M, N) or norm_weight.numel() != N:
        raise ValueError("linear_block_add_rmsnorm: resid must be [M, N] with unit inner stride, norm_weight [N]")
    lib = _lib.load()
    wsp, nbytes = _block_ws(lib, M, N, K, True, workspace)
    h = torch.empty((M, N), dtype=x.dtype, device=x.device)
    y = torch.empty((M, N), dtype=x.dtype, device=x.device)
    check(lib.md_linear_block_add_rmsnorm(_p(x), x.stride(0), _p(weight.data), _p(bias), _p(resid), resid.stride(0),
                                          _p(norm_weight), float(eps), _p(h), _p(y), M, N, K, wsp, nbytes, _stream()),
          "md_linear_block_add_rmsnorm")
    return h, y


# ----------------------------------------------------------------------------- K8b
FL_NONE, FL_SWIGLU, FL_RESID, FL_ROPE_APPEND, FL_XIELU, FL_GEGLU = 0, 1, 2, 3, 4, 5


def fused_linear_supported(M, N, K, epilogue=FL_NONE):
    """True when md_linear_fused (csrc/tilegemm.hip) takes this shape."""
    return bool(_lib.load().md_linear_fused_supported(int(M), int(N), int(K), int(epilogue)))


def _fused_args(x, weight: "PackedWeight", bias, epilogue):
    _gpu(x, weight.data, bias)
    if x.dim() != 2 or x.stride(1) != 1 or x.dtype != torch.bfloat16:
        raise ValueError("fused linear expects x [M, K] bf16 with unit inner stride")
    if weight.dtype != torch.bfloat16:
        raise TypeError("fused linear streams bf16 weights")
    M, K = x.shape
    if weight.K != K:
        raise ValueError(f"fused linear: x has K={K}, weight has K={weight.K}")
    if weight.swiglu != (epilogue in (FL_SWIGLU, FL_GEGLU)):
        raise ValueError("PackedWeight was packed for a different epilogue")
    a = _lib.FusedLinearArgs()
    a.x, a.ldx, a.w_packed, a.bias = x.data_ptr(), x.stride(0), weight.data.data_ptr(), (bias.data_ptr() if bias is not None else None)
    a.M, a.N, a.K, a.epilogue = M, weight.N, K, epilogue
    return a


def _run_fused(a):
    check(_lib.load().md_linear_fused(ctypes.byref(a), _stream()), "md_linear_fused")


class DeferredNorm:
    """An RMSNorm that has NOT been applied yet: `h` [M, K] are the un-normalised hidden states and `ssq` [M, K/32]
    the per-row partial sums of squares the residual epilogue of the producing linear wrote; the consuming fused
    linear normalises on the fly (md_linear_fused, deferred RMSNorm).  `materialize()` is the stand-alone kernel."""

    def __init__(self, h, ssq, weight, eps):
        self.h, self.ssq, self.weight, self.eps = h, ssq, weight, float(eps)

    def materialize(self):
        return rmsnorm(self.h, self.weight, self.eps)


def _set_pro(a, x, pro: "DeferredNorm"):
    if pro.h.data_ptr() != x.data_ptr() or pro.ssq.dtype != torch.float32 or not pro.ssq.is_contiguous():
        raise ValueError("deferred norm: x must be the un-normalised h the partial sums belong to")
    if (pro.ssq.dim() != 2 or pro.ssq.shape[0] != x.shape[0] or pro.ssq.shape[1] * 32 != x.shape[1]
            or pro.weight.numel() != x.shape[1] or pro.weight.dtype != torch.bfloat16):
        # ssq must hold one partial per 32-column tile of the producer (a shorter one would give a silently wrong rstd)
        raise ValueError("deferred norm: ssq [M, K / 32] float32 and a bf16 norm weight [K] expected")
    a.pro_ssq, a.pro_tiles = pro.ssq.data_ptr(), pro.ssq.shape[1]
    a.pro_norm_w, a.pro_eps = pro.weight.data_ptr(), pro.eps


def fused_linear(x, weight: "PackedWeight", bias=None, swiglu=False, resid=None, out=None, want_ssq=False,
                 pro: "DeferredNorm" = None, xielu=None, gelu=False):
    """One launch (md_linear_fused): F.linear(x, W, bias) for M <= 256 rows over a PackedWeight, optionally followed by
    SiLU(h1) * h3 (swiglu=True, weight = [w1; w3]) or by the bf16 residual add `resid + linear` (resid [M, N]).
    want_ssq (with resid): also return the per-row partial sums of squares [M, N/32] of the result (the producer half of
    a deferred RMSNorm).  pro (with swiglu): x is pro.h and is normalised on the fly (the consumer half)."""
    epi = FL_RESID if resid is not None else (FL_XIELU if xielu is not None else FL_NONE)
    if swiglu:
        epi = FL_GEGLU if gelu else FL_SWIGLU
    if xielu is not None and epi != FL_XIELU:
        raise ValueError("fused linear: the xIELU epilogue takes nothing beside it")
    a = _fused_args(x, weight, bias, epi)
    if xielu is not None:
        a.act = _act_numbers(xielu).value
    n_out = weight.N // 2 if swiglu else weight.N
    if out is None:
        out = torch.empty((x.shape[0], n_out), dtype=x.dtype, device=x.device)
    else:
        _gpu(out)
        if out.dtype != torch.bfloat16 or out.dim() != 2 or out.shape != (x.shape[0], n_out) or out.stride(1) != 1:
            raise ValueError("fused linear: out must be bf16 [M, N_out] with unit inner stride")
    a.out, a.ldo = out.data_ptr(), out.stride(0)
    ssq = None
    if resid is not None:
        _gpu(resid)
        if resid.shape != out.shape or resid.stride(1) != 1 or resid.dtype != torch.bfloat16:
            raise ValueError("fused linear: resid must be bf16 [M, N] with unit inner stride")
        a.resid, a.ldr = resid.data_ptr(), resid.stride(0)
        if want_ssq:
            ssq = torch.empty((x.shape[0], weight.N // 32), dtype=torch.float32, device=x.device)
            a.ssq_out = ssq.data_ptr()
    elif want_ssq:
        raise ValueError("fused linear: want_ssq belongs to the residual epilogue")
    if pro is not None:
        if not swiglu:
            raise ValueError("fused linear: the deferred-norm prologue exists for the w1|w3 and qkv linears")
        _set_pro(a, x, pro)
    _run_fused(a)
    return (out, ssq) if want_ssq else out


def fused_qkv_rope_append(x, weight: "PackedWeight", bias, H, KH, D, rows_per_req, offsets, table: RopeTable, kv_cache,
                          page_indices, page_indptr, last_page_len, kv_cache2=None, page_indices2=None,
                          page_indptr2=None, last_page_len2=None, kv_scales=None, kv_layout="NHD",
                          pro: "DeferredNorm" = None):
    """wqkv + RoPE + paged KV append in one launch (md_linear_fused, MD_FL_ROPE_APPEND): x [M, K] are the normalised
    hidden states of a decode / verify step in which request b owns rows [b * rows_per_req, (b+1) * rows_per_req).
    Returns the rotated q [M, H, D]; rotated k and v go to the paged cache (and to kv_cache2, bf16 NHD, when given).
    Same results as linear -> rope_append."""
    a = _fused_args(x, weight, bias, FL_ROPE_APPEND)
    _gpu(kv_cache, kv_cache2)
    M = x.shape[0]
    if weight.N != (H + 2 * KH) * D:
        raise ValueError("fused qkv: weight rows must be (H + 2 KH) * D")
    if M % rows_per_req:
        raise ValueError("fused qkv: every request must own rows_per_req rows")
    q_out = torch.empty((M, H, D), dtype=x.dtype, device=x.device)
    a.out, a.ldo = q_out.data_ptr(), H * D
    a.H, a.KH, a.D, a.rows_per_req, a.max_pos = H, KH, D, rows_per_req, table.max_pos
    offsets = _i32(offsets)
    pi, pp, lp = _i32(page_indices), _i32(page_indptr), _i32(last_page_len)
    a.offsets, a.cos_sin = offsets.data_ptr(), table.table.data_ptr()
    a.cache, a.page_indices, a.page_indptr, a.last_page_len = kv_cache.data_ptr(), pi.data_ptr(), pp.data_ptr(), lp.data_ptr()
    keep = [offsets, pi, pp, lp]
    if kv_cache2 is not None:
        pi2, pp2, lp2 = _i32(page_indices2), _i32(page_indptr2), _i32(last_page_len2)
        keep += [pi2, pp2, lp2]
        a.cache2, a.page_indices2, a.page_indptr2, a.last_page_len2 = (kv_cache2.data_ptr(), pi2.data_ptr(),
                                                                       pp2.data_ptr(), lp2.data_ptr())
    a.page_size = _kv_geom(kv_cache, kv_layout)[0]
    kvd, ks, vs = _kv_args(kv_cache, kv_scales, kv_layout)
    a.kv_dtype, a.k_scale, a.v_scale = kvd, ks, vs
    if pro is not None:                      # x is the un-normalised h: normalise on the fly (deferred RMSNorm)
        _set_pro(a, x, pro)
    _run_fused(a)
    return q_out


# ----------------------------------------------------------------------------- K9
def rmsnorm(x, weight, eps):
    _gpu(x, weight)
    dim = x.shape[-1]
    x2 = x.reshape(-1, dim)
    if not x2.is_contiguous():
        x2 = x2.contiguous()
    y = torch.empty_like(x2)
    lib = _lib.load()
    check(lib.md_rmsnorm(_p(x2), _p(weight), _p(y), x2.shape[0], dim, float(eps), _stream()), "md_rmsnorm")
    return y.view(x.shape)


def add_rmsnorm(x, r, weight, eps):
    """h = x + r ; y = rmsnorm(h).  Returns (h, y)."""
    _gpu(x, r, weight)
    dim = x.shape[-1]
    x2, r2 = x.reshape(-1, dim), r.reshape(-1, dim)
    if not x2.is_contiguous():
        x2 = x2.contiguous()
    if not r2.is_contiguous():
        r2 = r2.contiguous()
    h = torch.empty_like(x2)
    y = torch.empty_like(x2)
    lib = _lib.load()
    check(lib.md_add_rmsnorm(_p(x2), _p(r2), _p(weight), _p(h), _p(y), x2.shape[0], dim, float(eps), _stream()),
          "md_add_rmsnorm")
    return h.view(x.shape), y.view(x.shape)


def silu_mul(a, b):
    """bf16(silu(a)) * b for 2-D row-strided views (e.g. the two halves of a fused w1|w3 GEMM output)."""
    _gpu(a, b)
    if a.dim() != 2 or a.stride(1) != 1 or b.stride(1) != 1:
        raise ValueError("silu_mul expects 2-D tensors with unit inner stride")
    rows, dim = a.shape
    y = torch.empty((rows, dim), dtype=a.dtype, device=a.device)
    lib = _lib.load()
    check(lib.md_silu_mul(_p(a), _p(b), a.stride(0), b.stride(0), _p(y), rows, dim, _stream()), "md_silu_mul")
    return y


# ----------------------------------------------------------------------------- K11
MD_T_BF16, MD_T_F32 = 0, 1
_MODEL_DTYPES = {torch.bfloat16: MD_T_BF16, torch.float32: MD_T_F32}


def _model_dtype(t):
    if t.dtype not in _MODEL_DTYPES:
        raise TypeError(f"the layered decoder kernels take bfloat16 or float32 tensors, got {t.dtype}")
    return _MODEL_DTYPES[t.dtype]


def _dense(*ts):
    for t in ts:
        if t is not None and not t.is_contiguous():
            raise ValueError("expected contiguous tensors")


class StepRows:
    """Which rows a step runs: request b owns rows qo_indptr[b] .. qo_indptr[b+1]-1 at positions pos0[b] + 0, 1, ...;
    `slots[b]` is its entry in per-sequence state (None: b); n_max bounds the rows of one request (host)."""

    def __init__(self, qo_indptr, pos0, n_max, slots=None):
        self.qo_indptr, self.pos0, self.n_max, self.slots = _i32(qo_indptr), _i32(pos0), int(n_max), slots
        self.B = qo_indptr.numel() - 1
        if pos0.numel() < self.B or (slots is not None and slots.numel() < self.B):
            raise ValueError("StepRows: one position and one slot per request expected")
        if slots is not None:
            _i32(slots)


def embed_pos(tokens, table, pos_table, rows: StepRows, scale=1.0):
    """float32 residual rows E[token] * scale + P[pos] (pos_table may be None)."""
    _gpu(tokens, table, pos_table)
    _dense(tokens, table, pos_table)
    vocab, width = table.shape
    if tokens.dtype != torch.int64:
        raise TypeError("embed_pos: token ids are int64")
    if pos_table is not None and (pos_table.dtype != table.dtype or pos_table.shape[1] != width):
        raise ValueError("embed_pos: the position table must match the embedding table")
    out = torch.empty((tokens.numel(), width), dtype=torch.float32, device=table.device)
    check(_lib.load().md_embed_pos(_p(tokens), _p(table), _p(pos_table), _model_dtype(table), _p(rows.qo_indptr),
                                   _p(rows.pos0), rows.B, rows.n_max, width, vocab,
                                   pos_table.shape[0] if pos_table is not None else 1, float(scale), _p(out), _stream()),
          "md_embed_pos")
    return out


class Planes:
    """A projection as n fp32 partial planes [n, rows, width] in a workspace (a split-K product before its combine); valid
    until the next user of the workspace."""

    def __init__(self, planes):
        self.planes, self.n, self.shape = planes, planes.shape[0], tuple(planes.shape[1:])

    def sum(self):
        return self.planes.sum(0)


PLANES_KINDS = {"skinny": 0, "tile": 1, "block": 2}


def linear_planes_count(kind, M, N, K):
    """Partial planes of this product on the split-K GEMM `kind` (0: unsupported)."""
    return int(_lib.load().md_linear_planes_count(PLANES_KINDS[kind], int(M), int(N), int(K)))


def linear_planes(x, weight: "PackedWeight", kind, workspace: AttnWorkspace):
    """x . W^T as `Planes` in the workspace: one launch; resid_norm is the combine."""
    _gpu(x, weight.data)
    if x.dim() != 2 or x.stride(1) != 1 or x.dtype != torch.bfloat16 or weight.swiglu or weight.dtype != torch.bfloat16:
        raise ValueError("linear_planes expects bf16 x [M, K] with unit inner stride and a plain bf16 packed weight")
    M, K = x.shape
    if weight.K != K:
        raise ValueError(f"linear_planes: x has K={K}, weight has K={weight.K}")
    n = linear_planes_count(kind, M, weight.N, K)
    if n == 0:
        raise ValueError(f"linear_planes: {kind} does not take M={M} N={weight.N} K={K}")
    nbytes = n * M * weight.N * 4
    ws = workspace.get(nbytes + 256)
    off = (-ws.data_ptr()) % 256
    planes = ws[off:off + nbytes].view(torch.float32).view(n, M, weight.N)
    check(_lib.load().md_linear_planes(PLANES_KINDS[kind], _p(x), x.stride(0), _p(weight.data), M, weight.N, K, _p(planes),
                                       nbytes, _stream()), "md_linear_planes")
    return Planes(planes)


def resid_norm(x, delta, weight, eps, out_scale=1.0, shift=None, ring=None, rows: StepRows = None):
    """(x + delta, y): the fp32 residual add and the weighted RMS norm behind it, y in weight's dtype.  delta: rows of that
    dtype, `Planes`, or None (x is returned as it is).  shift [width] + ring [slots, R, width] float32: the token shift
    (md_resid_norm_shift); the ring is updated."""
    _gpu(x, weight, shift, ring)
    _dense(x, weight, shift, ring)
    M, width = x.shape
    if x.dtype != torch.float32 or weight.numel() != width:
        raise ValueError("resid_norm: x must be float32 [rows, width], weight [width]")
    a = _lib.ResidNormArgs()
    a.x, a.weight, a.rows, a.width = x.data_ptr(), weight.data_ptr(), M, width
    a.dtype, a.eps, a.out_scale = _model_dtype(weight), float(eps), float(out_scale)
    x_out = x
    if delta is not None:
        if tuple(delta.shape) != (M, width):
            raise ValueError(f"resid_norm: delta is {tuple(delta.shape)}, the residual {(M, width)}")
        x_out = torch.empty_like(x)
        a.x_out = x_out.data_ptr()
        if isinstance(delta, Planes):
            a.planes, a.n_planes = delta.planes.data_ptr(), delta.n
        else:
            _gpu(delta)
            _dense(delta)
            if delta.dtype != weight.dtype:
                raise TypeError("resid_norm: delta must have the weight's dtype")
            a.delta = delta.data_ptr()
    y = torch.empty((M, width), dtype=weight.dtype, device=x.device)
    a.y = y.data_ptr()
    lib = _lib.load()
    if shift is None:
        check(lib.md_resid_norm(ctypes.byref(a), _stream()), "md_resid_norm")
    else:
        if ring.dtype != torch.float32 or ring.dim() != 3 or ring.shape[2] != width or shift.dtype != weight.dtype:
            raise ValueError("resid_norm: ring must be float32 [slots, R, width], shift of the weight's dtype")
        a.shift, a.ring, a.ring_len = shift.data_ptr(), ring.data_ptr(), ring.shape[1]
        a.qo_indptr, a.pos0, a.B, a.n_max = rows.qo_indptr.data_ptr(), rows.pos0.data_ptr(), rows.B, rows.n_max
        a.slots = rows.slots.data_ptr() if rows.slots is not None else None
        check(lib.md_resid_norm_shift(ctypes.byref(a), _stream()), "md_resid_norm_shift")
    return x_out, y


def xielu(z, act, out=None):
    """xIELU of 2-D rows; act = float32 [2] on the device (the numbers in front of the softplus)."""
    _gpu(z, act)
    if z.dim() != 2 or z.stride(1) != 1 or act.dtype != torch.float32 or act.numel() != 2:
        raise ValueError("xielu expects 2-D rows with unit inner stride and float32 act[2]")
    y = torch.empty(z.shape, dtype=z.dtype, device=z.device) if out is None else out
    check(_lib.load().md_xielu(_p(z), z.stride(0), _p(act), _p(y), z.shape[0], z.shape[1], _model_dtype(z), _stream()),
          "md_xielu")
    return y


def head_pad(head_size):
    """Width the extended attention's pages and queries are padded to."""
    n = int(_lib.load().md_xattn_head_pad(int(head_size)))
    if n == 0:
        raise ValueError(f"head size {head_size} unsupported")
    return n


class XattnSpec:
    """The constants of one extended-attention layer (md_xattn_args): heads, sizes, score scale, chunk (0: none), softmax
    sink, query/key norm, and the per-head distance bias r1, r2 (float32 [H] or None).  score_bound: see magicdec_hip.h."""

    def __init__(self, H, KH, D, DV, scale, eps, chunk=0, sink=False, qk_norm=False, r1=None, r2=None, score_bound=0.0):
        self.H, self.KH, self.D, self.DV = int(H), int(KH), int(D), int(DV)
        self.scale, self.eps, self.chunk = float(scale), float(eps), int(chunk)
        self.sink, self.qk_norm, self.score_bound = bool(sink), bool(qk_norm), float(score_bound)
        for r in (r1, r2):
            if r is not None and (r.dtype != torch.float32 or r.numel() != self.H or not r.is_contiguous()):
                raise ValueError("distance bias: float32 [H] expected")
        self.r1, self.r2 = r1, r2


def _xattn_args(s: XattnSpec, k_cache, v_cache, rows: StepRows, page_indices, page_indptr, max_pages, dtype):
    _gpu(k_cache, v_cache)
    _dense(k_cache, v_cache)
    if k_cache.dim() != 4 or k_cache.shape[:3] != v_cache.shape[:3] or k_cache.shape[1] != s.KH:
        raise ValueError("extended attention: pages must be [pages, KH, page_size, width]")
    if k_cache.shape[3] != head_pad(s.D) or v_cache.shape[3] != head_pad(s.DV) or k_cache.dtype != dtype:
        raise ValueError("extended attention: pages of another head size or dtype")
    if page_indptr.numel() != rows.B + 1:
        raise ValueError("extended attention: page table of another batch")
    a = _lib.XattnArgs()
    a.k_cache, a.v_cache = k_cache.data_ptr(), v_cache.data_ptr()
    a.qo_indptr, a.pos0, a.B, a.n_max = rows.qo_indptr.data_ptr(), rows.pos0.data_ptr(), rows.B, rows.n_max
    a.page_indices, a.page_indptr = _i32(page_indices).data_ptr(), _i32(page_indptr).data_ptr()
    a.page_size, a.max_pages = k_cache.shape[2], int(max_pages)
    a.H, a.KH, a.D, a.DV, a.scale, a.eps = s.H, s.KH, s.D, s.DV, s.scale, s.eps
    a.chunk, a.sink, a.qk_norm, a.score_bound = s.chunk, int(s.sink), int(s.qk_norm), s.score_bound
    a.r1 = s.r1.data_ptr() if s.r1 is not None else None
    a.r2 = s.r2.data_ptr() if s.r2 is not None else None
    a.dtype = _MODEL_DTYPES[dtype]
    return a


def extended_attention(qkv, s: XattnSpec, k_cache, v_cache, rows: StepRows, page_indices, page_indptr, max_pages,
                       workspace: AttnWorkspace, fuse=True, plain=False):
    """One attention layer over the raw projection rows qkv [M, H*D + KH*D + KH*DV]: normalise q and k, append k and v,
    attend.  Returns [M, H * DV].  Decode / verify steps are one launch where md_xattn_fused_supported (fuse=False: the
    separate normalise + append launch); plain=True forces the plain attention kernel (comparison)."""
    _gpu(qkv)
    M = qkv.shape[0]
    if qkv.dim() != 2 or qkv.stride(1) != 1 or qkv.shape[1] != (s.H + s.KH) * s.D + s.KH * s.DV:
        raise ValueError("extended attention: qkv rows must be q | k | v heads")
    lib = _lib.load()
    a = _xattn_args(s, k_cache, v_cache, rows, page_indices, page_indptr, max_pages, qkv.dtype)
    a.qkv, a.ld_qkv = qkv.data_ptr(), qkv.stride(0)
    out = torch.empty((M, s.H * s.DV), dtype=qkv.dtype, device=qkv.device)
    a.out, a.force_plain = out.data_ptr(), int(plain)
    q = None
    if (plain or not fuse or qkv.stride(0) % 8 or qkv.data_ptr() % 16 or not lib.md_xattn_fused_supported(ctypes.byref(a))):
        q = torch.empty((M, s.H, k_cache.shape[3]), dtype=qkv.dtype, device=qkv.device)
        check(lib.md_qk_norm_append(ctypes.byref(a), _p(q), _stream()), "md_qk_norm_append")
        a.q = q.data_ptr()
    nbytes = lib.md_xattn_workspace_bytes(ctypes.byref(a))
    if nbytes and not plain:
        ws = workspace.get(nbytes + 256)
        off = (-ws.data_ptr()) % 256
        a.workspace, a.workspace_bytes = ws.data_ptr() + off, nbytes
    check(lib.md_xattn(ctypes.byref(a), _stream()), "md_xattn")
    return out


# ----------------------------------------------------------------------------- K12
class RotaryTable:
    """(cos, sin) of every position and neighbouring pair, float32 [max_pos, dims / 2, 2], computed in float64 on the host.
    base^(-2i / dims) with optional YaRN scaling (factor, original, fast, slow): frequencies below `slow` turns over the original
    length are divided by the factor, those above `fast` turns stay, a linear ramp between; the amplitude is 1 + ln(factor) / 10."""

    def __init__(self, dims, base, max_pos, scaling=None, device="cuda"):
        if dims <= 0 or dims % 2:
            raise ValueError(f"rotary positions: {dims} dimensions do not form pairs")
        i = torch.arange(dims // 2, dtype=torch.float64)
        freq, amp = base ** (-2.0 * i / dims), 1.0
        if scaling is not None:
            factor, original, fast, slow = scaling

            def index(turns):
                return dims * math.log(original / (2 * math.pi * turns)) / (2 * math.log(base))
            lo, hi = max(math.floor(index(fast)), 0), min(math.ceil(index(slow)), dims - 1)
            ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0, 1)
            freq, amp = freq / factor * ramp + freq * (1 - ramp), 0.1 * math.log(factor) + 1.0
        ang = torch.arange(max_pos, dtype=torch.float64).view(-1, 1) * freq
        self.table = (torch.stack([ang.cos(), ang.sin()], -1) * amp).float().contiguous().to(device)
        self.max_pos, self.pairs = int(max_pos), dims // 2


def latent_row_width(kv_rank, rot_dim):
    """Elements of a latent cache row: latent, rotated key part, padding."""
    n = int(_lib.load().md_latent_row_width(int(kv_rank), int(rot_dim)))
    if n == 0:
        raise ValueError(f"latent size {kv_rank} with a rotated part of {rot_dim} is unsupported")
    return n


class LatentSpec:
    """The constants of one latent-attention layer (md_latent_args): heads, sizes, score scale, rotation, and its weights in the
    kernels' layouts: absorb [H, kv_rank, dim] (keys, moved to the query), expand [H * (dim + vdim), kv_rank] (keys, then values),
    values [H, vdim, kv_rank] (a view of expand's second part)."""

    def __init__(self, H, dim, rot_dim, vdim, q_rank, kv_rank, scale, eps, rotary: RotaryTable, expand, dq_norm, kv_norm=None):
        self.H, self.dim, self.rot_dim, self.vdim = int(H), int(dim), int(rot_dim), int(vdim)
        self.q_rank, self.kv_rank, self.scale, self.eps, self.rotary = int(q_rank), int(kv_rank), float(scale), float(eps), rotary
        self.width = latent_row_width(kv_rank, rot_dim)
        if tuple(expand.shape) != (H * (dim + vdim), kv_rank) or not expand.is_contiguous() or 2 * rotary.pairs > rot_dim:
            raise ValueError("latent attention: expand must be [H * (dim + vdim), kv_rank], the rotation within rot_dim")
        self.expand, self.dq_norm, self.kv_norm = expand, dq_norm, kv_norm
        self.absorb = expand[:H * dim].view(H, dim, kv_rank).transpose(1, 2).contiguous()
        self.values = expand[H * dim:].view(H, vdim, kv_rank)

    def flops(self, new, ctx):
        """(absorbed, expanded) multiply-adds per head for `new` rows per request at the end of `ctx` positions (host lists):
        which form of the attention a step should take."""
        R = self.kv_rank
        pairs = sum(n * (c - (n - 1) / 2) for n, c in zip(new, ctx))
        absorbed = pairs * (2 * R + self.rot_dim) + sum(new) * R * (self.dim + self.vdim)
        expanded = pairs * (self.dim + self.rot_dim + self.vdim) + sum(ctx) * R * (self.dim + self.vdim)
        return absorbed, expanded


def _latent_args(s: LatentSpec, cache, rows: StepRows, page_indices, page_indptr, max_pages, dtype):
    _gpu(cache)
    _dense(cache)
    if cache.dim() != 3 or cache.shape[2] != s.width or cache.dtype != dtype:
        raise ValueError("latent attention: pages must be [pages, page_size, row width] of the model's dtype")
    if page_indptr.numel() != rows.B + 1:
        raise ValueError("latent attention: page table of another batch")
    a = _lib.LatentArgs()
    a.cache, a.cos_sin, a.max_pos, a.rot_pairs = cache.data_ptr(), s.rotary.table.data_ptr(), s.rotary.max_pos, s.rotary.pairs
    a.qo_indptr, a.pos0, a.B, a.n_max = rows.qo_indptr.data_ptr(), rows.pos0.data_ptr(), rows.B, rows.n_max
    a.page_indices, a.page_indptr = _i32(page_indices).data_ptr(), _i32(page_indptr).data_ptr()
    a.page_size, a.max_pages = cache.shape[1], int(max_pages)
    a.H, a.dim, a.rot_dim, a.vdim, a.q_rank, a.kv_rank = s.H, s.dim, s.rot_dim, s.vdim, s.q_rank, s.kv_rank
    a.scale, a.eps, a.dtype = s.scale, s.eps, _MODEL_DTYPES[dtype]
    return a


def latent_append(z, s: LatentSpec, cache, rows: StepRows, page_indices, page_indptr, max_pages):
    """z [M, >= q_rank (+ kv_rank + rot_dim)]: the normalised query latents [M, q_rank]; with s.kv_norm the normalised latent and
    the rotated key part of every row go to its position's cache row."""
    _gpu(z)
    if z.dim() != 2 or z.stride(1) != 1 or z.shape[1] < s.q_rank + (s.kv_rank + s.rot_dim if s.kv_norm is not None else 0):
        raise ValueError("latent_append: rows must hold the query latent, the latent and the key part")
    a = _latent_args(s, cache, rows, page_indices, page_indptr, max_pages, z.dtype)
    cq = torch.empty((z.shape[0], s.q_rank), dtype=z.dtype, device=z.device)
    a.z, a.ldz, a.cq, a.dq_norm = z.data_ptr(), z.stride(0), cq.data_ptr(), s.dq_norm.data_ptr()
    if s.kv_norm is not None:
        a.kv_norm, a.append = s.kv_norm.data_ptr(), 1
    check(_lib.load().md_latent_append(ctypes.byref(a), _stream()), "md_latent_append")
    return cq


def head_linear(x, w, out, gate=None):
    """out[:, h] = x[:, h] . w[h]^T (* sigmoid(gate[:, h])) for x [M, H, K], w [H, N, K], out [M, H, >= N] (strides free in the
    first two dimensions)."""
    _head_linear(x, w, out, gate)
    return out


def _head_linear(x, w, out, gate=None, tail=None, tail_pad=0, rotary=None, rows=None):
    _gpu(x, w, out, gate, tail)
    _dense(w)
    M, H, K = x.shape
    if w.dim() != 3 or w.shape[0] != H or w.shape[2] != K or tuple(out.shape[:2]) != (M, H):
        raise ValueError(f"head_linear: x {tuple(x.shape)}, w {tuple(w.shape)}, out {tuple(out.shape)}")
    for t in (x, out) + ((tail,) if tail is not None else ()) + ((gate,) if gate is not None else ()):
        if t.stride(-1) != 1 or t.dtype != w.dtype:
            raise ValueError("head_linear: unit inner strides and one dtype expected")
    a = _lib.HeadLinearArgs()
    a.x, a.w, a.out = x.data_ptr(), w.data_ptr(), out.data_ptr()
    a.ldx, a.hx, a.ldo, a.ho = x.stride(0), x.stride(1), out.stride(0), out.stride(1)
    a.M, a.H, a.N, a.K, a.dtype = M, H, w.shape[1], K, _model_dtype(w)
    if out.shape[2] < a.N + tail_pad:
        raise ValueError("head_linear: out is too narrow")
    if gate is not None:
        if tuple(gate.shape) != (M, H):
            raise ValueError("head_linear: gate must be [rows, heads]")
        a.gate, a.ld_gate = gate.data_ptr(), gate.stride(0)
    if tail is not None:
        a.tail, a.ldt, a.ht, a.tail_dim, a.tail_pad = tail.data_ptr(), tail.stride(0), tail.stride(1), tail.shape[2], tail_pad
        a.cos_sin, a.max_pos, a.rot_pairs = rotary.table.data_ptr(), rotary.max_pos, rotary.pairs
        a.qo_indptr, a.pos0, a.B = rows.qo_indptr.data_ptr(), rows.pos0.data_ptr(), rows.B
    check(_lib.load().md_head_linear(ctypes.byref(a), _stream()), "md_head_linear")


def latent_attention(q, s: LatentSpec, cache, rows: StepRows, page_indices, page_indptr, max_pages, workspace: AttnWorkspace, out,
                     gate=None, ctx=None, plain=False):
    """out [M, H, vdim] (row stride free) = softmax attention of q [M, H * (dim + rot_dim)] (as projected) over the cache, which
    latent_append has brought up to the step's own rows, times sigmoid(gate [M, H]).  ctx = `LatentContext`: the expanded form is
    taken where it is cheaper; without it, in 32-bit or for unusual sizes the absorbed form.  plain: its plain kernel."""
    _gpu(q, out)
    M = q.shape[0]
    if tuple(q.shape) != (M, s.H * (s.dim + s.rot_dim)) or not q.is_contiguous() or tuple(out.shape) != (M, s.H, s.vdim):
        raise ValueError("latent attention: q must be [rows, H * (dim + rot_dim)], out [rows, H, vdim]")
    if out.stride(2) != 1 or out.stride(1) != s.vdim or (gate is not None and gate.stride(1) != 1):
        raise ValueError("latent attention: heads of out must be dense")
    lib = _lib.load()
    a = _latent_args(s, cache, rows, page_indices, page_indptr, max_pages, q.dtype)
    a.force_plain = int(plain)
    if (ctx is not None and not plain and ctx.expanded(s) and out.stride(0) % 4 == 0 and out.data_ptr() % 8 == 0
            and lib.md_latent_prefill_supported(ctypes.byref(a))):
        dense = torch.empty((ctx.total, s.kv_rank), dtype=q.dtype, device=q.device)
        a.ctx_indptr = ctx.indptr.data_ptr()
        check(lib.md_latent_gather(ctypes.byref(a), ctx.longest, _p(dense), _stream()), "md_latent_gather")
        kv = torch.nn.functional.linear(dense, s.expand)
        a.q, a.kv, a.out, a.ldo = q.data_ptr(), kv.data_ptr(), out.data_ptr(), out.stride(0)
        if gate is not None:
            a.gate, a.ld_gate = gate.data_ptr(), gate.stride(0)
        check(lib.md_latent_prefill(ctypes.byref(a), _stream()), "md_latent_prefill")
        return out
    heads = q.view(M, s.H, s.dim + s.rot_dim)
    qa = torch.empty((M, s.H, s.width), dtype=q.dtype, device=q.device)
    _head_linear(heads[..., :s.dim], s.absorb, qa, tail=heads[..., s.dim:], tail_pad=s.width - s.kv_rank, rotary=s.rotary,
                 rows=rows)
    lat = torch.empty((M, s.H, s.kv_rank), dtype=q.dtype, device=q.device)
    a.q, a.out = qa.data_ptr(), lat.data_ptr()
    nbytes = lib.md_latent_workspace_bytes(ctypes.byref(a))
    if nbytes:
        ws = workspace.get(nbytes + 256)
        a.workspace, a.workspace_bytes = ws.data_ptr() + (-ws.data_ptr()) % 256, nbytes
    check(lib.md_latent_attn(ctypes.byref(a), _stream()), "md_latent_attn")
    _head_linear(lat, s.values, out, gate=gate)
    return out


class LatentContext:
    """What the host knows of a step's requests: `new` rows each, at the end of `ctx` positions."""
    MAX_EXPANDED_BYTES = 24 << 30

    def __init__(self, new, ctx, device):
        self.new, self.ctx, self.total, self.longest = list(new), list(ctx), sum(ctx), max(ctx)
        self._device, self._indptr, self._choice = device, None, {}

    @property
    def indptr(self):
        if self._indptr is None:
            at = [0]
            for c in self.ctx:
                at.append(at[-1] + c)
            self._indptr = torch.tensor(at, dtype=torch.int32).to(self._device)
        return self._indptr

    def expanded(self, s: LatentSpec):
        """Does the expanded form take fewer operations (and fit) for these requests?"""
        key = (s.H, s.dim, s.rot_dim, s.vdim, s.kv_rank)
        if key not in self._choice:
            absorbed, expanded = s.flops(self.new, self.ctx)
            size = self.total * s.H * (s.dim + s.vdim) * 2
            self._choice[key] = expanded < absorbed and max(self.new) >= 64 and size <= self.MAX_EXPANDED_BYTES
        return self._choice[key]


def embed_bigram(tokens, table, pairs, norm_weight, eps, mul_before, mul_token, history, rows: StepRows, page_indices, page_indptr):
    """float32 rows rms(table[t] + pairs[(mul_before * before + mul_token * t) mod n]) * norm_weight; the last row of `pairs`
    (row n) for a sequence's first token.  history: int32 [pages, page_size], the tokens of every sequence by position."""
    _gpu(tokens, table, pairs, norm_weight, history)
    _dense(tokens, table, pairs, norm_weight, history)
    vocab, width = table.shape
    if tokens.dtype != torch.int64 or history.dtype != torch.int32 or history.dim() != 2:
        raise TypeError("embed_bigram: token ids are int64, the token history int32 [pages, page_size]")
    if pairs.shape[1] != width or pairs.shape[0] < 2 or norm_weight.numel() != width or not (pairs.dtype == norm_weight.dtype == table.dtype):
        raise ValueError("embed_bigram: tables of different widths or dtypes")
    if page_indptr.numel() != rows.B + 1:
        raise ValueError("embed_bigram: page table of another batch")
    out = torch.empty((tokens.numel(), width), dtype=torch.float32, device=table.device)
    check(_lib.load().md_embed_bigram(_p(tokens), _p(table), _p(pairs), _p(norm_weight), _model_dtype(table), _p(rows.qo_indptr),
                                      _p(rows.pos0), rows.B, rows.n_max, width, vocab, pairs.shape[0] - 1, int(mul_before),
                                      int(mul_token), _p(history), _p(_i32(page_indices)), _p(_i32(page_indptr)), history.shape[1],
                                      float(eps), _p(out), _stream()), "md_embed_bigram")
    return out


def gelu_mul(a, b, out=None):
    """gelu_tanh(a) * b of 2-D rows with unit inner stride (fp32, one rounding)."""
    _gpu(a, b, out)
    if a.dim() != 2 or a.shape != b.shape or a.stride(1) != 1 or b.stride(1) != 1 or a.dtype != b.dtype:
        raise ValueError("gelu_mul expects 2-D rows of one shape with unit inner stride")
    y = torch.empty(a.shape, dtype=a.dtype, device=a.device) if out is None else out
    if y.shape != a.shape or y.stride(1) != 1 or y.dtype != a.dtype:
        raise ValueError("gelu_mul: out of another shape or dtype")
    check(_lib.load().md_gelu_mul(_p(a), _p(b), a.stride(0), b.stride(0), _p(y), y.stride(0), a.shape[0], a.shape[1], _model_dtype(a),
                                  _stream()), "md_gelu_mul")
    return y


def softcap_(z, cap):
    """cap * tanh(z / cap) of 2-D rows, in place."""
    _gpu(z)
    if z.dim() != 2 or z.stride(1) != 1:
        raise ValueError("softcap_ expects 2-D rows with unit inner stride")
    check(_lib.load().md_softcap(_p(z), z.stride(0), float(cap), z.shape[0], z.shape[1], _model_dtype(z), _stream()), "md_softcap")
    return z


# ----------------------------------------------------------------------------- K10
def argmax(logits, index_offset=0, return_values=False):
    """Row-wise argmax of bf16 (or float32) logits [rows, vocab] (lowest index among equal maxima)."""
    _gpu(logits)
    if logits.dim() != 2 or logits.stride(1) != 1:
        raise ValueError("argmax expects [rows, vocab] with unit inner stride")
    rows, vocab = logits.shape
    idx = torch.empty(rows, dtype=torch.int64, device=logits.device)
    if logits.dtype == torch.float32:
        if return_values or index_offset:
            raise ValueError("argmax: values and index offsets exist for bf16 logits")
        check(_lib.load().md_argmax_f32(_p(logits), logits.stride(0), rows, vocab, _p(idx), _stream()), "md_argmax_f32")
        return idx
    vals = torch.empty(rows, dtype=logits.dtype, device=logits.device) if return_values else None
    lib = _lib.load()
    check(lib.md_argmax(_p(logits), logits.stride(0), rows, vocab, int(index_offset), _p(vals), _p(idx), _stream()),
          "md_argmax")
    return (vals, idx) if return_values else idx


def argmax_tp_slots(logits, tp_rank, tp_world, index_offset=0):
    """(vals [rows, tp_world] bf16, idx [rows, tp_world] int64): the row-wise argmax of this rank's vocab shard in column
    tp_rank, zeros elsewhere -- the tensors the reference sum-all-reduces before its merge (Engine/SnapKV/model.py:178-184),
    written by the argmax launch itself."""
    _gpu(logits)
    if logits.dim() != 2 or logits.stride(1) != 1:
        raise ValueError("argmax_tp_slots expects [rows, vocab] with unit inner stride")
    rows, vocab = logits.shape
    vals = torch.empty((rows, tp_world), dtype=logits.dtype, device=logits.device)
    idx = torch.empty((rows, tp_world), dtype=torch.int64, device=logits.device)
    check(_lib.load().md_argmax_tp_slots(_p(logits), logits.stride(0), rows, vocab, int(index_offset), int(tp_rank),
                                         int(tp_world), _p(vals), _p(idx), _stream()), "md_argmax_tp_slots")
    return vals, idx


def tp_argmax_merge(vals, idx):
    """vals [rows, tp] bf16, idx [rows, tp] int64 -> winning global index per row (lowest rank on ties)."""
    _gpu(vals, idx)
    rows, tp = vals.shape
    out = torch.empty(rows, dtype=torch.int64, device=vals.device)
    lib = _lib.load()
    check(lib.md_tp_argmax_merge(_p(vals.contiguous()), _p(idx.contiguous()), rows, tp, _p(out), _stream()),
          "md_tp_argmax_merge")
    return out


# ----------------------------------------------------------------------------- a1
def accept_rollback(tokens_buffer, target_tokens, output, num_nodes, cachelens, last_page_len, draft_cachelens,
                    draft_last_page_len, gamma, draft_rollback, draft_cap, eot_1, eot_2, max_nodes, accept_nums,
                    bonus, double_buffer, cachelens_update, flags):
    """The verify-loop body (tests/SnapKV/longspec_benchmark.py:208-285) as one launch; all tensors are
    updated in place, `flags` = int32[2] (terminal, next_double)."""
    _gpu(tokens_buffer, target_tokens, output, num_nodes, cachelens, last_page_len)
    B = tokens_buffer.shape[0]
    lib = _lib.load()
    check(lib.md_accept_rollback(_p(tokens_buffer), _p(target_tokens), _p(output), output.shape[1], _p(num_nodes),
                                 _p(cachelens), _p(last_page_len), _p(draft_cachelens), _p(draft_last_page_len), B,
                                 gamma, draft_rollback, draft_cap, int(eot_1), int(eot_2), int(max_nodes),
                                 _p(accept_nums), _p(bonus), _p(double_buffer), _p(cachelens_update), _p(flags),
                                 _stream()), "md_accept_rollback")
