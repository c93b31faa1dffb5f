"""Operators of the section of the C ABI for hybrid decoders (norms around sublayers, attention, recurrences, experts)
(include/muillm_amd.h), in the manner of muillm_ext.py: validate, allocate outputs with torch, hand raw
pointers and the current stream to the library. Activations and weights are fp16, bf16 or fp32 tensors of
one dtype; the residual stream, router logits, recurrence gates and state are fp32."""

from __future__ import annotations

import ctypes
from dataclasses import dataclass
from typing import List, Optional, Tuple

import torch

from . import _lib
from ._lib import MUI_DTYPE_BF16, MUI_DTYPE_F16, MUI_DTYPE_F32, check

_CODES = {torch.float16: MUI_DTYPE_F16, torch.bfloat16: MUI_DTYPE_BF16, torch.float32: MUI_DTYPE_F32}


def dtype_code(dtype: torch.dtype) -> int:
    code = _CODES.get(dtype)
    if code is None:
        raise ValueError(f"unsupported dtype {dtype}: fp16, bf16 or fp32")
    return code


def _ptr(t: Optional[torch.Tensor]) -> Optional[int]:
    return None if t is None else t.data_ptr()


def _stream(t: torch.Tensor) -> int:
    return torch.cuda.current_stream(t.device).cuda_stream


def _operand(t: Optional[torch.Tensor], name: str, like: torch.Tensor, shape=None, dtype=None) -> None:
    """What a raw pointer needs: contiguous, on the activations' device, of the expected type and shape."""
    if t is None:
        return
    want = like.dtype if dtype is None else dtype
    if not t.is_cuda or t.device != like.device:
        raise RuntimeError(f"{name} must be a CUDA tensor on {like.device}")
    if t.dtype != want or not t.is_contiguous():
        raise RuntimeError(f"{name} must be a contiguous {want} tensor")
    if shape is not None and tuple(t.shape) != tuple(shape):
        raise RuntimeError(f"{name} has shape {tuple(t.shape)}, expected {tuple(shape)}")


def _positions(cache_position: torch.Tensor, row_start: Optional[torch.Tensor], like: torch.Tensor, batch: int, t: int) -> None:
    _operand(cache_position, "cache_position", like, (t,), torch.int64)
    _operand(row_start, "row_start", like, (batch,), torch.int64)


# --------------------------------------------------------------------------------------
# residual stream
# --------------------------------------------------------------------------------------
@dataclass
class MoEOutput:
    """A mixture of experts whose weighted sum is taken where it joins the residual stream."""
    pairs: torch.Tensor     # [tokens * top, width]
    identity: torch.Tensor  # [tokens, width]
    expert: torch.Tensor    # int32 [tokens, top]
    weight: torch.Tensor    # fp32 [tokens, top]
    n_experts: int

    def dense(self) -> torch.Tensor:
        """The weighted sum as an fp32 tensor [tokens, width]."""
        tokens, top = self.expert.shape
        x = residual_norm(None, self, None, None, 0.0)[0]
        return x.reshape(tokens, -1)


def residual_norm(residual: Optional[torch.Tensor], y, post_gain: Optional[torch.Tensor],
                  next_gain: Optional[torch.Tensor], eps: float, y_scale: float = 1.0, branch_scale: float = 1.0,
                  next_scale: float = 1.0, emit: bool = False) -> Tuple[torch.Tensor, Optional[torch.Tensor]]:
    """(residual + branch_scale norm_post(y), next_scale norm_next of that): the boundary between two sublayers.
    residual fp32 [..., width] or None (zero), updated in place; y a tensor [..., width] or a MoEOutput; a gain
    that is None skips its norm: without post_gain y_scale * y joins as it is, without next_gain the second
    result is the (scaled) sum itself, rounded, where emit asks for it, and None otherwise."""
    moe = isinstance(y, MoEOutput)
    src = y.identity if moe else y
    width = src.shape[-1]
    rows = src.numel() // width
    if not src.is_contiguous():
        src = src.contiguous()
    if not src.is_cuda:
        raise RuntimeError("residual_norm needs CUDA tensors")
    out = torch.empty(src.shape, dtype=torch.float32, device=src.device) if residual is None else residual
    _operand(residual, "residual", src, None, torch.float32)
    if residual is not None and residual.numel() != src.numel():
        raise RuntimeError("residual and sublayer output differ in size")
    _operand(post_gain, "post_gain", src, (width,))
    _operand(next_gain, "next_gain", src, (width,))
    h = torch.empty_like(src) if emit or next_gain is not None else None
    if rows == 0:
        return out, h
    lib, code = _lib.load(), dtype_code(src.dtype)
    if moe:
        tokens, top = y.expert.shape
        _operand(y.pairs, "pairs", src, (tokens * top, width))
        _operand(y.expert, "expert", src, (rows, top), torch.int32)
        _operand(y.weight, "weight", src, (rows, top), torch.float32)
        check(lib.mui_moe_residual_norm(_stream(src), code, _ptr(residual), y.pairs.data_ptr(), src.data_ptr(),
                                        y.expert.data_ptr(), y.weight.data_ptr(), y.n_experts, top, _ptr(post_gain),
                                        float(branch_scale), _ptr(next_gain), float(next_scale), float(eps), out.data_ptr(),
                                        _ptr(h), rows, width), "mui_moe_residual_norm")
    else:
        check(lib.mui_residual_norm(_stream(src), code, _ptr(residual), src.data_ptr(), float(y_scale), _ptr(post_gain),
                                    float(branch_scale), _ptr(next_gain), float(next_scale), float(eps), out.data_ptr(), _ptr(h),
                                    rows, width), "mui_residual_norm")
    return out, h


def linear_f32(x: torch.Tensor, weight: torch.Tensor, bias: Optional[torch.Tensor] = None) -> torch.Tensor:
    """fp32 [tokens, n] = x W^T + bias for x [..., k]: outputs that stay in 32 bits (router logits, gates)."""
    n, k = weight.shape
    if x.shape[-1] != k:
        raise RuntimeError(f"input has {x.shape[-1]} features but the weights expect {k}")
    x = x.contiguous()
    _operand(weight, "weight", x)
    _operand(bias, "bias", x, (n,))
    tokens = x.numel() // k
    y = torch.empty((tokens, n), dtype=torch.float32, device=x.device)
    check(_lib.load().mui_linear_f32(_stream(x), dtype_code(x.dtype), weight.data_ptr(), x.data_ptr(), _ptr(bias),
                                     y.data_ptr(), n, k, tokens), "mui_linear_f32")
    return y


# --------------------------------------------------------------------------------------
# mixture of experts
# --------------------------------------------------------------------------------------
def moe_route(logits: torch.Tensor, correction: Optional[torch.Tensor], n_experts: int, top: int, tile_pairs: int):
    """(expert int32 [T, top], weight fp32 [T, top], pairs, tiles): see mui_moe_route. logits fp32
    [T, outputs]; outputs beyond n_experts are identity experts."""
    tokens, n_out = logits.shape
    _operand(logits, "logits", logits, None, torch.float32)
    dtype = logits.dtype if correction is None else correction.dtype
    _operand(correction, "correction", logits, (n_out,), dtype)
    lib, dev = _lib.load(), logits.device
    expert = torch.empty((tokens, top), dtype=torch.int32, device=dev)
    weight = torch.empty((tokens, top), dtype=torch.float32, device=dev)
    pairs = tiles = None
    if tile_pairs:
        pairs = torch.empty(tokens * top, dtype=torch.int32, device=dev)
        n_tiles = lib.mui_moe_max_tiles(tokens, top, n_experts, tile_pairs)
        tiles = torch.empty((n_tiles + 1, 4), dtype=torch.int32, device=dev)
    check(lib.mui_moe_route(_stream(logits), dtype_code(dtype), logits.data_ptr(), _ptr(correction), n_experts,
                            n_out - n_experts, top, tokens, tile_pairs, expert.data_ptr(), weight.data_ptr(),
                            _ptr(pairs), _ptr(tiles)), "mui_moe_route")
    return expert, weight, pairs, tiles


def moe_experts(x: torch.Tensor, gate: torch.Tensor, up: torch.Tensor, down: torch.Tensor, limit: float, expert, pairs,
                tiles, tile_pairs: int) -> torch.Tensor:
    """[T * top, width]: every chosen expert's output (rows of identity experts are not written).
    gate, up [E, ff, width], down [E, width, ff]."""
    n_experts, ff, width = gate.shape
    tokens, top = expert.shape
    _operand(x, "x", x, (tokens, width))
    _operand(gate, "gate", x)
    _operand(up, "up", x, (n_experts, ff, width))
    _operand(down, "down", x, (n_experts, width, ff))
    lib, code, st = _lib.load(), dtype_code(x.dtype), _stream(x)
    act = torch.empty((tokens * top, ff), dtype=x.dtype, device=x.device)
    out = torch.empty((tokens * top, width), dtype=x.dtype, device=x.device)
    check(lib.mui_moe_gateup(st, code, gate.data_ptr(), up.data_ptr(), ff * width, x.data_ptr(), float(limit),
                             expert.data_ptr(), _ptr(pairs), _ptr(tiles), tile_pairs, act.data_ptr(), n_experts, ff,
                             width, top, tokens), "mui_moe_gateup")
    check(lib.mui_moe_down(st, code, down.data_ptr(), width * ff, act.data_ptr(), expert.data_ptr(), _ptr(pairs),
                           _ptr(tiles), tile_pairs, out.data_ptr(), n_experts, width, ff, top, tokens), "mui_moe_down")
    return out


def moe_tile_pairs(dtype: torch.dtype, tokens: int, top: int, n_experts: int, width: int, ff: int) -> int:
    return _lib.load().mui_moe_tile_pairs(dtype_code(dtype), tokens, top, n_experts, width, ff)


# --------------------------------------------------------------------------------------
# latent attention
# --------------------------------------------------------------------------------------
def latent_prepare(down: torch.Tensor, q_gain: torch.Tensor, kv_gain: Optional[torch.Tensor], eps: float,
                   inv_freq: torch.Tensor, cache_position: torch.Tensor, row_start: Optional[torch.Tensor],
                   c_cache: torch.Tensor, r_cache: torch.Tensor):
    """(query latent [B, T, q_rank], cos_sin fp32 [B * T, rot]); with kv_gain the tokens' latent rows and
    rotated key parts go to their cache slots. down [B, T, q_rank (+ kv_rank + rot)]; caches [B, capacity, .]."""
    b, t = down.shape[0], down.shape[1]
    q_rank, kv_rank, rot = q_gain.numel(), c_cache.shape[-1], r_cache.shape[-1]
    _operand(down, "down", down, (b, t, q_rank + (kv_rank + rot if kv_gain is not None else 0)))
    _operand(q_gain, "q_gain", down)
    _operand(kv_gain, "kv_gain", down, (kv_rank,))
    _operand(inv_freq, "inv_freq", down, (rot // 2,), torch.float64)
    _operand(c_cache, "c_cache", down)
    _operand(r_cache, "r_cache", down, (c_cache.shape[0], c_cache.shape[1], rot))
    _positions(cache_position, row_start, down, b, t)
    if b > c_cache.shape[0]:
        raise RuntimeError("more batch rows than the cache has")
    q_latent = torch.empty((b, t, q_rank), dtype=down.dtype, device=down.device)
    cos_sin = torch.empty((b * t, rot), dtype=torch.float32, device=down.device)
    check(_lib.load().mui_latent_prepare(_stream(down), dtype_code(down.dtype), down.data_ptr(), down.shape[-1],
                                         q_gain.data_ptr(), _ptr(kv_gain), float(eps), inv_freq.data_ptr(),
                                         cache_position.data_ptr(), _ptr(row_start), q_latent.data_ptr(),
                                         cos_sin.data_ptr(), c_cache.data_ptr(), c_cache.stride(0), r_cache.data_ptr(),
                                         r_cache.stride(0), b, t, q_rank, kv_rank, rot, c_cache.shape[1]),
          "mui_latent_prepare")
    return q_latent, cos_sin


def latent_route(dtype: torch.dtype, tokens: int, heads: int, dim: int, rot: int, vdim: int, kv_rank: int) -> int:
    return _lib.load().mui_latent_attention_route(dtype_code(dtype), tokens, heads, dim, rot, vdim, kv_rank)


def _check_latent(q, cos_sin, heads, dim, rot):
    b, t = q.shape[0], q.shape[1]
    _operand(q, "q", q, (b, t, heads * (dim + rot)))
    _operand(cos_sin, "cos_sin", q, (b * t, rot), torch.float32)
    return b, t


def latent_attention(q: torch.Tensor, cos_sin: torch.Tensor, w_uk: torch.Tensor, w_uv: torch.Tensor, c_cache: torch.Tensor,
                     r_cache: torch.Tensor, cache_position: torch.Tensor, row_start: Optional[torch.Tensor], heads: int,
                     dim: int, vdim: int, scale: float, window: int, route: int) -> torch.Tensor:
    """Attention of q [B, T, heads * (dim + rot)] (unrotated as projected) over the latent caches, which hold
    the new tokens already: [B, T, heads * vdim]."""
    kv_rank, rot, cap = c_cache.shape[-1], r_cache.shape[-1], c_cache.shape[1]
    b, t = _check_latent(q, cos_sin, heads, dim, rot)
    _operand(w_uk, "w_uk", q, (heads * dim, kv_rank))
    _operand(w_uv, "w_uv", q, (heads * vdim, kv_rank))
    _operand(c_cache, "c_cache", q)
    _operand(r_cache, "r_cache", q)
    _positions(cache_position, row_start, q, b, t)
    if b > c_cache.shape[0]:
        raise RuntimeError("more batch rows than the cache has")
    lib = _lib.load()
    out = torch.empty((b, t, heads * vdim), dtype=q.dtype, device=q.device)
    span = min(window, cap) if window > 0 else cap
    scratch = None
    if route == _lib.MUI_LATENT_DECODE:
        nbytes = lib.mui_latent_decode_scratch_bytes(b, t, heads, kv_rank, rot, span)
        scratch = torch.empty(nbytes, dtype=torch.uint8, device=q.device)
    check(lib.mui_latent_attention(_stream(q), dtype_code(q.dtype), route, q.data_ptr(), cos_sin.data_ptr(),
                                   w_uk.data_ptr(), w_uv.data_ptr(), c_cache.data_ptr(), c_cache.stride(0),
                                   r_cache.data_ptr(), r_cache.stride(0), cache_position.data_ptr(), _ptr(row_start),
                                   float(scale), int(window), _ptr(scratch), span, out.data_ptr(), b, t, heads, dim, rot,
                                   vdim, kv_rank, cap), "mui_latent_attention")
    return out


def latent_prefill_attention(q: torch.Tensor, cos_sin: torch.Tensor, kv: List[torch.Tensor], kv_first: int,
                             r_cache: torch.Tensor, row_start: Optional[torch.Tensor], q_first: int, heads: int, dim: int,
                             vdim: int, scale: float, window: int) -> torch.Tensor:
    """The same for a prompt (or a portion of one) with the keys and values of slots kv_first .. made
    beforehand: kv[b] = [rows, heads * (dim | vdim)] per batch row."""
    rot = r_cache.shape[-1]
    b, t = _check_latent(q, cos_sin, heads, dim, rot)
    _operand(r_cache, "r_cache", q)
    _operand(row_start, "row_start", q, (b,), torch.int64)
    rows = q_first + t - kv_first
    if q_first + t > r_cache.shape[1] or b > r_cache.shape[0]:
        raise RuntimeError("the tokens lie outside the cache")
    lib = _lib.load()
    out = torch.empty((b, t, heads * vdim), dtype=q.dtype, device=q.device)
    for i in range(b):
        _operand(kv[i], "kv", q, (rows, heads * (dim + vdim)))
        check(lib.mui_latent_prefill_attention(_stream(q), dtype_code(q.dtype), q.data_ptr(), cos_sin.data_ptr(),
                                               kv[i].data_ptr(), kv_first, rows, r_cache.data_ptr(), r_cache.stride(0),
                                               _ptr(row_start), float(scale), int(window), q_first, out.data_ptr(), i, t,
                                               heads, dim, rot, vdim), "mui_latent_prefill_attention")
    return out


# --------------------------------------------------------------------------------------
# matrix-memory recurrence
# --------------------------------------------------------------------------------------
def mlstm_slices(dv: int) -> int:
    return _lib.load().mui_mlstm_slices(dv)


MLSTM_SEGMENT = 4096  # tokens per call: bounds the workspace of a long prompt


def mlstm(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, gates: torch.Tensor, state, q_scale: float, gate_cap: float,
          cache_position: torch.Tensor, row_start: Optional[torch.Tensor], heads: int) -> torch.Tensor:
    """o fp32 [B, T, heads, dv]; advances state = (S, n, m) in place. q, k [B, T, heads * dk] and v
    [B, T, heads * dv] may be column slices of one projection's output; gates fp32 [B, T, 2 * heads]."""
    b, t = q.shape[0], q.shape[1]
    dk, dv = q.shape[2] // heads, v.shape[2] // heads
    pitch = q.stride(1)
    for name, x in (("q", q), ("k", k), ("v", v)):
        if not x.is_cuda or x.dtype != q.dtype or x.stride(2) != 1 or x.stride(1) != pitch or (b > 1 and x.stride(0) != t * pitch):
            raise RuntimeError(f"{name} must be a slice of a contiguous [B, T, .] projection output")
    s, n, m = state
    slices = mlstm_slices(dv)
    _operand(gates, "gates", q, (b, t, 2 * heads), torch.float32)
    for name, x, shape in (("S", s, (heads, dk, dv)), ("n", n, (heads, slices, dk)), ("m", m, (heads, slices))):
        _operand(x, name, q, (x.shape[0],) + shape, torch.float32)
        if x.shape[0] < b:
            raise RuntimeError("more batch rows than the state has")
    _positions(cache_position, row_start, q, b, t)
    o = torch.empty((b, t, heads, dv), dtype=torch.float32, device=q.device)
    lib = _lib.load()
    if t > MLSTM_SEGMENT and b > 1:  # (the kernels address a whole batch by one token count)
        return torch.cat([mlstm(q[i:i + 1], k[i:i + 1], v[i:i + 1], gates[i:i + 1], tuple(x[i:i + 1] for x in state),
                                q_scale, gate_cap, cache_position, None if row_start is None else row_start[i:i + 1],
                                heads) for i in range(b)])
    for t0 in range(0, t, MLSTM_SEGMENT):
        tn = min(MLSTM_SEGMENT, t - t0)
        nbytes = lib.mui_mlstm_workspace_bytes(b, tn, heads, dk, dv)
        ws = torch.empty(nbytes, dtype=torch.uint8, device=q.device) if nbytes else None
        check(lib.mui_mlstm(_stream(q), dtype_code(q.dtype), q[:, t0:].data_ptr(), k[:, t0:].data_ptr(),
                            v[:, t0:].data_ptr(), pitch, gates[:, t0:].data_ptr(), float(q_scale), float(gate_cap),
                            s.data_ptr(), n.data_ptr(), m.data_ptr(), cache_position[t0:].data_ptr(), _ptr(row_start),
                            o[:, t0:].data_ptr(), _ptr(ws), b, tn, heads, dk, dv), "mui_mlstm")
    return o


def mlstm_output(o: torch.Tensor, gain: torch.Tensor, gate: torch.Tensor, eps: float) -> torch.Tensor:
    """[B, T, heads * dv] in gate's dtype: o over its head's root mean square, times gain and sigmoid(gate)."""
    b, t, heads, dv = o.shape
    _operand(o, "o", gate, None, torch.float32)
    _operand(gain, "gain", gate, (heads * dv,))
    if gate.stride(2) != 1 or (b > 1 and gate.stride(0) != t * gate.stride(1)):
        raise RuntimeError("gate must be a slice of a contiguous [B, T, .] projection output")
    y = torch.empty((b, t, heads * dv), dtype=gate.dtype, device=gate.device)
    check(_lib.load().mui_mlstm_output(_stream(gate), dtype_code(gate.dtype), o.data_ptr(), gain.data_ptr(),
                                       gate.data_ptr(), gate.stride(1), float(eps), y.data_ptr(), b * t, heads, dv),
          "mui_mlstm_output")
    return y


# --------------------------------------------------------------------------------------
# token plus bigram embedding
# --------------------------------------------------------------------------------------
def bigram_embedding(ids: torch.Tensor, prev: torch.Tensor, cache_position: torch.Tensor, row_start: Optional[torch.Tensor],
                     table: torch.Tensor, bigram: torch.Tensor, scale: float, mul_prev: int, mul_cur: int):
    """(x fp32, h in the table's dtype) [B, T, width]: scale * table row + bigram row of (previous, current) token; prev
    int64 [B'] holds the ids in front of this call's first tokens and takes its last ones. bigram [buckets + 1, width]."""
    b, t = ids.shape
    vocab, width = table.shape
    ids = ids.to(torch.int64).contiguous()
    _operand(table, "table", table)
    _operand(bigram, "bigram", table, (bigram.shape[0], width))
    _operand(ids, "ids", table, None, torch.int64)
    _operand(prev, "prev", table, None, torch.int64)
    _positions(cache_position, row_start, table, b, t)
    if b > prev.numel():
        raise RuntimeError("more batch rows than the state has")
    x = torch.empty((b, t, width), dtype=torch.float32, device=table.device)
    h = torch.empty((b, t, width), dtype=table.dtype, device=table.device)
    check(_lib.load().mui_bigram_embedding(_stream(table), dtype_code(table.dtype), ids.data_ptr(), prev.data_ptr(),
                                           cache_position.data_ptr(), _ptr(row_start), table.data_ptr(), bigram.data_ptr(),
                                           float(scale), mul_prev, mul_cur, bigram.shape[0] - 1, x.data_ptr(), h.data_ptr(),
                                           b, t, width, vocab), "mui_bigram_embedding")
    return x, h


# --------------------------------------------------------------------------------------
# grouped-query attention over cached rows
# --------------------------------------------------------------------------------------
def hybrid_prepare(proj: torch.Tensor, heads: int, kv_heads: int, dim: int, vdim: int, q_gain: Optional[torch.Tensor],
                   k_gain: Optional[torch.Tensor], eps: float, inv_freq: torch.Tensor, cache_position: torch.Tensor,
                   row_start: Optional[torch.Tensor], k_cache: torch.Tensor, v_cache: torch.Tensor) -> torch.Tensor:
    """Normed and rotated queries [B, T, heads * dim]; keys and values go to their cache slots. proj [B, T, .] starts
    with q | k | v; caches [B', capacity, kv_heads * dim | kv_heads * vdim]; inv_freq double [rotated dims / 2]."""
    b, t, pitch = proj.shape
    nq, nk, nv = heads * dim, kv_heads * dim, kv_heads * vdim
    if pitch < nq + nk + nv:
        raise RuntimeError("the projection has too few columns")
    _operand(proj, "proj", proj)
    _operand(q_gain, "q_gain", proj, (nq,))
    _operand(k_gain, "k_gain", proj, (nk,))
    _operand(inv_freq, "inv_freq", proj, None, torch.float64)
    _operand(k_cache, "k_cache", proj, (k_cache.shape[0], k_cache.shape[1], nk))
    _operand(v_cache, "v_cache", proj, (k_cache.shape[0], k_cache.shape[1], nv))
    _positions(cache_position, row_start, proj, b, t)
    if b > k_cache.shape[0]:
        raise RuntimeError("more batch rows than the cache has")
    q = torch.empty((b, t, nq), dtype=proj.dtype, device=proj.device)
    check(_lib.load().mui_hybrid_prepare(_stream(proj), dtype_code(proj.dtype), proj.data_ptr(), pitch, nq, nq + nk, _ptr(q_gain),
                                         _ptr(k_gain), float(eps), inv_freq.data_ptr(), 2 * inv_freq.numel(),
                                         cache_position.data_ptr(), _ptr(row_start), q.data_ptr(), k_cache.data_ptr(),
                                         k_cache.stride(0), v_cache.data_ptr(), v_cache.stride(0), b, t, heads, kv_heads, dim,
                                         vdim, k_cache.shape[1]), "mui_hybrid_prepare")
    return q


def hybrid_route(dtype: torch.dtype, tokens: int, dim: int, vdim: int) -> int:
    return _lib.load().mui_hybrid_attention_route(dtype_code(dtype), tokens, dim, vdim)


def hybrid_attention(q: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor, gate: Optional[torch.Tensor],
                     cache_position: torch.Tensor, row_start: Optional[torch.Tensor], heads: int, kv_heads: int, scale: float,
                     softcap: float = 0.0, window: int = 0, keep_first: int = 0, route: Optional[int] = None) -> torch.Tensor:
    """[B, T, heads * vdim]: attention of q [B, T, heads * dim] over the caches, which hold the new tokens already, times
    sigmoid(gate); gate: a column slice [B, T, heads * vdim] of a projection's output, or None."""
    b, t = q.shape[0], q.shape[1]
    cap, dim, vdim = k_cache.shape[1], k_cache.shape[2] // kv_heads, v_cache.shape[2] // kv_heads
    _operand(q, "q", q, (b, t, heads * dim))
    _operand(k_cache, "k_cache", q, (k_cache.shape[0], cap, kv_heads * dim))
    _operand(v_cache, "v_cache", q, (k_cache.shape[0], cap, kv_heads * vdim))
    _positions(cache_position, row_start, q, b, t)
    if b > k_cache.shape[0]:
        raise RuntimeError("more batch rows than the cache has")
    pitch = 0
    if gate is not None:
        pitch = gate.stride(1)
        if not gate.is_cuda or gate.dtype != q.dtype or tuple(gate.shape) != (b, t, heads * vdim) or gate.stride(2) != 1 or \
                (b > 1 and gate.stride(0) != t * pitch):
            raise RuntimeError("gate must be a slice of a contiguous [B, T, .] projection output")
    lib = _lib.load()
    if route is None:
        route = hybrid_route(q.dtype, t, dim, vdim)
    if route != _lib.MUI_HYBRID_PLAIN and gate is not None and (pitch % 4 or gate.data_ptr() % 8):
        route = _lib.MUI_HYBRID_PLAIN
    out = torch.empty((b, t, heads * vdim), dtype=q.dtype, device=q.device)
    span = min(window + keep_first, cap) if window > 0 else cap
    scratch = None
    if route == _lib.MUI_HYBRID_DECODE:
        nbytes = lib.mui_hybrid_decode_scratch_bytes(b, t, heads, kv_heads, vdim, span)
        scratch = torch.empty(nbytes, dtype=torch.uint8, device=q.device) if nbytes else None
    check(lib.mui_hybrid_attention(_stream(q), dtype_code(q.dtype), route, q.data_ptr(), k_cache.data_ptr(), k_cache.stride(0),
                                   v_cache.data_ptr(), v_cache.stride(0), _ptr(gate), pitch, cache_position.data_ptr(),
                                   _ptr(row_start), float(scale), float(softcap), window, keep_first, _ptr(scratch), span,
                                   out.data_ptr(), b, t, heads, kv_heads, dim, vdim, cap), "mui_hybrid_attention")
    return out


# --------------------------------------------------------------------------------------
# gated delta rule
# --------------------------------------------------------------------------------------
DELTA_SEGMENT = 4096  # tokens per call: bounds the workspace of a long prompt


@dataclass
class ChannelDelta:
    """One layer's constants and parameters; offsets: columns of q, k, v, a, g, b in the projection's output."""
    heads: int
    kv_heads: int
    dk: int
    dv: int
    offsets: Tuple[int, int, int, int, int, int]
    conv: torch.Tensor     # [2 kv_heads dk + heads dv, taps]
    a2: torch.Tensor       # [heads * dk, ra]
    dt_bias: torch.Tensor  # [heads * dk]
    a_log: torch.Tensor    # [heads]
    g2: torch.Tensor       # [heads * dv, rg]
    gain: torch.Tensor     # [dv]
    eps: float

    @property
    def channels(self) -> int:
        return 2 * self.kv_heads * self.dk + self.heads * self.dv

    @property
    def ring_rows(self) -> int:
        return _lib.load().mui_channel_delta_ring_rows(self.conv.shape[1])

    def descriptor(self) -> "_lib.MuiChannelDeltaDesc":
        ptrs = [x.data_ptr() for x in (self.conv, self.a2, self.dt_bias, self.a_log, self.g2, self.gain)]
        return _lib.MuiChannelDeltaDesc(*ptrs, self.heads, self.kv_heads, self.dk, self.dv, self.a2.shape[1], self.g2.shape[1],
                                        self.conv.shape[1], *self.offsets, self.dk ** -0.5, self.eps)


def channel_delta(layer: ChannelDelta, proj: torch.Tensor, state: torch.Tensor, ring: torch.Tensor,
                  cache_position: torch.Tensor, row_start: Optional[torch.Tensor]) -> torch.Tensor:
    """y [B, T, heads * dv] of the projection's output proj [B, T, .]; advances state fp32 [B', heads, dk, dv] and the ring
    of the convolutions' inputs [B', ring_rows, channels] in place."""
    b, t, pitch = proj.shape
    c = layer
    _operand(proj, "proj", proj)
    _operand(c.conv, "conv", proj, (c.channels, c.conv.shape[1]))
    _operand(c.a2, "a2", proj, (c.heads * c.dk, c.a2.shape[1]))
    _operand(c.dt_bias, "dt_bias", proj, (c.heads * c.dk,))
    _operand(c.a_log, "a_log", proj, (c.heads,))
    _operand(c.g2, "g2", proj, (c.heads * c.dv, c.g2.shape[1]))
    _operand(c.gain, "gain", proj, (c.dv,))
    _operand(state, "state", proj, (state.shape[0], c.heads, c.dk, c.dv), torch.float32)
    _operand(ring, "ring", proj, (state.shape[0], c.ring_rows, c.channels))
    _positions(cache_position, row_start, proj, b, t)
    if b > state.shape[0]:
        raise RuntimeError("more batch rows than the state has")
    lib = _lib.load()
    most = min(DELTA_SEGMENT, lib.mui_channel_delta_max_tokens(c.dk, c.conv.shape[1]))
    if t > most and b > 1:  # (the kernels address a whole batch by one token count)
        return torch.cat([channel_delta(layer, proj[i:i + 1], state[i:i + 1], ring[i:i + 1], cache_position,
                                        None if row_start is None else row_start[i:i + 1]) for i in range(b)])
    y = torch.empty((b, t, c.heads * c.dv), dtype=proj.dtype, device=proj.device)
    desc = c.descriptor()
    for t0 in range(0, t, most):
        tn = min(most, t - t0)
        nbytes = lib.mui_channel_delta_workspace_bytes(b, tn, c.heads, c.dk, c.dv) if tn > _lib.MUI_MAX_TOKENS else 0
        ws = torch.empty(nbytes, dtype=torch.uint8, device=proj.device) if nbytes else None
        check(lib.mui_channel_delta(_stream(proj), dtype_code(proj.dtype), ctypes.byref(desc), proj[:, t0:].data_ptr(), pitch, state.data_ptr(),
                                    ring.data_ptr(), cache_position[t0:].data_ptr(), _ptr(row_start), y[:, t0:].data_ptr(),
                                    _ptr(ws), b, tn), "mui_channel_delta")
    return y
