"""Host wrappers of the row, attention and recurrence kernels in libsocket_core.so
(csrc/rows.hip, csrc/chunk_attend.hip, csrc/latent.hip, csrc/recurrence.hip).

The residual stream of these models is fp32; activations, projections and caches
have the model's dtype (bf16 or fp32).  A sublayer's output is handed on as a
`Pending` and added to the stream by the launch that computes the next norm.  Where a
design averages a layer's result with earlier ones (`Depth`), that launch, or in a decode
step the output product itself, does so too.
"""
from __future__ import annotations

import ctypes
from dataclasses import dataclass
from typing import Optional, Tuple

import torch
from torch import Tensor
from torch.nn import functional as F

from ._lib import (ChunkAttention, DepthMix, Latent, LatentAttend, Recurrence, Residual, RopeHalf, RowsLinear, check, core, dtype_enum, ptr, stream_ptr)

MAX_GEMV_ROWS = 4
GATED_UNITS = {"clamped": 1, "silu": 2}


@dataclass
class Depth:
    """What goes on after a layer is w[n] times its result plus the sum of w[j] * past[j] over the n
    results before it; the result is kept as past[n].  past [layers + 1, ..., dim] fp32."""
    past: Tensor
    n: int
    w: Tensor

    def struct(self) -> DepthMix:
        assert self.w.dtype == torch.float32 and self.w.numel() == self.n + 1 and self.w.is_contiguous()
        assert self.past.dtype == torch.float32 and self.past.is_contiguous() and self.past.shape[0] > self.n
        return DepthMix(past=self.past.data_ptr(), past_stride=self.past.stride(0), w=self.w.data_ptr(), n=self.n,
                        result=self.past[self.n].data_ptr())


@dataclass
class Pending:
    """A sublayer's output that is not in the residual stream yet: scale_a * a (+ scale_b * b),
    normalised with `post_w` on its way in (None: added as it is).  `depth`: the sum is a layer's
    result, averaged with earlier ones before it goes on."""
    a: Tensor
    scale_a: float = 1.0
    b: Optional[Tensor] = None
    scale_b: float = 0.0
    post_w: Optional[Tensor] = None
    depth: Optional[Depth] = None


def _row_stride(x: Tensor) -> int:
    """Elements between the rows of x [..., dim], whose rows are evenly spaced."""
    assert x.stride(-1) == 1
    step, rows = 0, 1
    for i in reversed(range(x.dim() - 1)):
        if x.shape[i] > 1:
            step = step or x.stride(i)
            assert x.stride(i) == step * rows, "rows are not evenly spaced"
            rows *= x.shape[i]
    return step or x.shape[-1]


def _residual(x: Optional[Tensor], embed, ids, pending: Optional[Pending], pre_w: Tensor, eps: float, dtype,
              x_out: Optional[Tensor], h_out: Optional[Tensor], embed_scale: float = 1.0) -> Residual:
    r = Residual(embed_scale=embed_scale)
    dim = pre_w.numel()
    assert pre_w.is_cuda and pre_w.dtype == torch.float32 and pre_w.is_contiguous()
    if x is not None:
        assert x.dtype == torch.float32 and x.shape[-1] == dim
        stride = _row_stride(x)
        r.x, r.x_stride = x.data_ptr(), 0 if stride == dim else stride
    else:
        assert embed.is_contiguous() and embed.dtype == dtype and embed.shape[1] == dim
        assert ids.is_contiguous() and ids.dtype in (torch.int32, torch.int64)
        r.embed, r.ids, r.ids64, r.vocab = embed.data_ptr(), ids.data_ptr(), int(ids.dtype == torch.int64), embed.shape[0]
    if pending is not None:
        for t in (pending.a, pending.b):
            assert t is None or (t.is_contiguous() and t.dtype == pending.a.dtype and t.shape[-1] == dim)
        r.a, r.scale_a, r.scale_b = pending.a.data_ptr(), pending.scale_a, pending.scale_b
        r.b = None if pending.b is None else pending.b.data_ptr()
        r.pending_f32 = int(pending.a.dtype == torch.float32)
        if pending.post_w is not None:
            assert pending.post_w.dtype == torch.float32 and pending.post_w.numel() == dim
            r.post_w = pending.post_w.data_ptr()
        if pending.depth is not None:
            r.depth = pending.depth.struct()
    r.pre_w, r.eps, r.dtype, r.dim = pre_w.data_ptr(), eps, dtype_enum(dtype), dim
    r.x_out = None if x_out is None else x_out.data_ptr()
    r.h_out = None if h_out is None else h_out.data_ptr()
    return r


def _stream_out(x, pending, lead, dim: int, device, x_out: Optional[Tensor]) -> Tensor:
    if x_out is not None:
        assert x_out.dtype == torch.float32 and x_out.is_contiguous() and tuple(x_out.shape) == (*lead, dim)
        return x_out
    return x if x is not None and pending is None else torch.empty(*lead, dim, dtype=torch.float32, device=device)


@torch.no_grad()
def residual_norm(x: Optional[Tensor], pending: Optional[Pending], pre_w: Tensor, eps: float, dtype, *,
                  embed: Optional[Tensor] = None, ids: Optional[Tensor] = None, embed_scale: float = 1.0,
                  x_out: Optional[Tensor] = None) -> Tuple[Tensor, Tensor]:
    """(x', h): x' = x + norm(pending) in fp32 (averaged over depth where pending asks for it),
    h = norm(x') in `dtype`.  With `x` None the stream starts at the rows `ids` of `embed`, times
    embed_scale.  `x_out`: where x' goes."""
    lead = x.shape[:-1] if x is not None else ids.shape
    dim = pre_w.numel()
    h = torch.empty(*lead, dim, dtype=dtype, device=pre_w.device)
    x_out = _stream_out(x, pending, lead, dim, pre_w.device, x_out)
    r = _residual(x, embed, ids, pending, pre_w, eps, dtype, None if x_out is x else x_out, h, embed_scale)
    check("socket_residual_norm", core().socket_residual_norm(ctypes.byref(r), h.numel() // dim, stream_ptr(h.device)))
    return x_out, h


def _gemv_fits(rows: int, x_dtype, weight: Tensor, limit: int) -> bool:
    return (rows <= limit and x_dtype == torch.bfloat16 and weight.dtype == torch.bfloat16
            and weight.shape[1] % 8 == 0 and weight.is_contiguous())


@torch.no_grad()
def linear_f32(x: Tensor, weight: Tensor) -> Tensor:
    """x @ weight.T with the 32-bit sums kept."""
    rows, K, N = x.numel() // x.shape[-1], x.shape[-1], weight.shape[0]
    if x.dtype == torch.float32:
        return F.linear(x, weight)
    if _gemv_fits(rows, x.dtype, weight, MAX_GEMV_ROWS) and x.is_contiguous():
        y = torch.empty(*x.shape[:-1], N, dtype=torch.float32, device=x.device)
        a = RowsLinear(x1=x.data_ptr(), w1=weight.data_ptr(), s1=1.0, K1=K, y=y.data_ptr(), y_f32=1, M=rows, N=N)
        check("socket_rows_linear_bf16", core().socket_rows_linear_bf16(ctypes.byref(a), stream_ptr(x.device)))
        return y
    return torch.mm(x.reshape(rows, K), weight.t(), out_dtype=torch.float32).view(*x.shape[:-1], N)


@torch.no_grad()
def norm_linear(x: Optional[Tensor], pending: Optional[Pending], pre_w: Tensor, eps: float, weight: Tensor, *,
                embed: Optional[Tensor] = None, ids: Optional[Tensor] = None, f32_out: bool = False,
                up_weight: Optional[Tensor] = None, act: str = "clamped", limit: float = 0.0,
                bias: Optional[Tensor] = None, up_bias: Optional[Tensor] = None, embed_scale: float = 1.0,
                x_out: Optional[Tensor] = None) -> Tuple[Tensor, Tensor]:
    """(x', y) for the few rows of a decode step: `residual_norm`, then y = h @ weight.T + bias, or
    with `up_weight` the gated unit of both products.  One launch where the matrix-vector
    kernel takes the shape."""
    dtype = weight.dtype
    lead = x.shape[:-1] if x is not None else ids.shape
    rows, K, N = 1, weight.shape[1], weight.shape[0]
    for n in lead:
        rows *= n
    if not _gemv_fits(rows, dtype, weight, MAX_GEMV_ROWS) or K > 16384 or (pending is not None and pending.depth is not None):
        x_out, h = residual_norm(x, pending, pre_w, eps, dtype, embed=embed, ids=ids, embed_scale=embed_scale, x_out=x_out)
        if up_weight is not None:
            return x_out, gated_unit(torch.cat([F.linear(h, weight, bias), F.linear(h, up_weight, up_bias)], dim=-1), act, limit)
        assert bias is None or not f32_out
        return x_out, linear_f32(h, weight) if f32_out else F.linear(h, weight, bias)
    x_out = _stream_out(x, pending, lead, K, weight.device, x_out)
    r = _residual(x, embed, ids, pending, pre_w, eps, dtype, None if x_out is x else x_out, None, embed_scale)
    y = torch.empty(*lead, N, dtype=torch.float32 if f32_out else dtype, device=weight.device)
    a = RowsLinear(norm=ctypes.pointer(r), w1=weight.data_ptr(), s1=1.0, K1=K, y=y.data_ptr(), y_f32=int(f32_out),
                   M=rows, N=N)
    if up_weight is not None:
        assert up_weight.shape == weight.shape and up_weight.is_contiguous() and up_weight.dtype == dtype
        a.w2, a.kind, a.limit = up_weight.data_ptr(), GATED_UNITS[act], limit
    a.b1, a.b2 = _bias(bias, N, dtype), _bias(up_bias, N, dtype)
    check("socket_rows_linear_bf16", core().socket_rows_linear_bf16(ctypes.byref(a), stream_ptr(weight.device)))
    return x_out, y


def _bias(b: Optional[Tensor], n: int, dtype):
    assert b is None or (b.numel() == n and b.dtype == dtype and b.is_contiguous())
    return None if b is None else b.data_ptr()


@torch.no_grad()
def linear_residual(h: Tensor, weight: Tensor, x: Tensor, bias: Optional[Tensor] = None,
                    depth: Optional[Depth] = None) -> Tuple[Tensor, Optional[Pending]]:
    """A sublayer's output product added to the stream x, with the average over depth, for the few
    rows of a decode step: (x', None) from one launch where the matrix-vector kernel takes the
    shape, else (x, the output as a Pending)."""
    rows, K, N = h.numel() // h.shape[-1], h.shape[-1], weight.shape[0]
    if not (_gemv_fits(rows, h.dtype, weight, MAX_GEMV_ROWS) and h.is_contiguous()):
        return x, Pending(F.linear(h, weight, bias), depth=depth)
    assert x.dtype == torch.float32 and x.is_contiguous() and x.numel() == rows * N
    y = torch.empty(*h.shape[:-1], N, dtype=torch.float32, device=h.device)
    a = RowsLinear(x1=h.data_ptr(), w1=weight.data_ptr(), s1=1.0, K1=K, y=y.data_ptr(), y_f32=1, M=rows, N=N,
                   b1=_bias(bias, N, weight.dtype), res=x.data_ptr())
    if depth is not None:
        a.depth = depth.struct()
    check("socket_rows_linear_bf16", core().socket_rows_linear_bf16(ctypes.byref(a), stream_ptr(h.device)))
    return y, None


@torch.no_grad()
def linear_terms(terms, rows_limit: int = MAX_GEMV_ROWS) -> Pending:
    """The sublayer output sum of scale * (x @ weight.T) over one or two (x, weight, scale)
    terms.  A decode step's rows give one fp32 tensor in one launch; others a tensor per
    term, whose sum the next norm's launch takes."""
    x, w, s = terms[0]
    rows, K = x.numel() // x.shape[-1], x.shape[-1]
    if all(_gemv_fits(rows, t.dtype, wt, rows_limit) and t.is_contiguous() for t, wt, _ in terms):
        y = torch.empty(*x.shape[:-1], w.shape[0], dtype=torch.float32, device=x.device)
        a = RowsLinear(x1=x.data_ptr(), w1=w.data_ptr(), s1=s, K1=K, y=y.data_ptr(), y_f32=1, M=rows, N=w.shape[0])
        if len(terms) == 2:
            x2, w2, s2 = terms[1]
            assert w2.shape[0] == w.shape[0]
            a.x2, a.w2, a.s2, a.K2 = x2.data_ptr(), w2.data_ptr(), s2, x2.shape[-1]
        check("socket_rows_linear_bf16", core().socket_rows_linear_bf16(ctypes.byref(a), stream_ptr(x.device)))
        return Pending(y)
    out = Pending(F.linear(x, w), s)
    if len(terms) == 2:
        out.b, out.scale_b = F.linear(terms[1][0], terms[1][1]), terms[1][2]
    return out


@torch.no_grad()
def gated_unit(gu: Tensor, act: str, limit: float = 0.0) -> Tensor:
    """Of the halves g, u of the last dimension: "clamped": g * sigmoid(1.702 g) * (u + 1) with g and u
    clamped at `limit`; "silu": g * sigmoid(g) * u."""
    assert gu.is_cuda and gu.is_contiguous()
    ff = gu.shape[-1] // 2
    out = torch.empty(*gu.shape[:-1], ff, dtype=gu.dtype, device=gu.device)
    check("socket_gated_unit", core().socket_gated_unit(ptr(gu), ptr(out), dtype_enum(gu.dtype), out.numel() // ff, ff,
                                                        GATED_UNITS[act], limit, stream_ptr(gu.device)))
    return out


@torch.no_grad()
def rope_half(proj: Tensor, q_off: int, k_off: int, H: int, G: int, D: int, rot_dims: int, cos_sin: Tensor, *,
              pos0: int = 0, pos: Optional[Tensor] = None, ring=None, q_pitch: int = 0):
    """Rotate the q and k heads in the rows proj [B,T,N].  Portion (pos None): (q [B,T,H,D],
    k [B,T,G,D]).  One token at the device position `pos`: the key goes into `ring`
    (a ChunkRing), returned is q [B,1,H,q_pitch]."""
    B, T, _ = proj.shape
    pitch = q_pitch or D
    q = torch.empty(B, T, H, pitch, dtype=proj.dtype, device=proj.device)
    k = None
    a = RopeHalf(proj=proj.data_ptr(), dtype=dtype_enum(proj.dtype), proj_stride_b=proj.stride(0),
                 proj_stride_t=proj.stride(1), q_off=q_off, k_off=k_off, H=H, G=G, D=D, rot_dims=rot_dims,
                 cos_sin=cos_sin.data_ptr(), n_pos=cos_sin.shape[0], pos0=pos0, q_out=q.data_ptr(), q_pitch=pitch, B=B, T=T,
                 chunk=1)
    assert proj.stride(2) == 1 and cos_sin.dtype == torch.float32 and cos_sin.is_contiguous()
    if pos is None:
        k = torch.empty(B, T, G, D, dtype=proj.dtype, device=proj.device)
        a.k_out = k.data_ptr()
    else:
        assert pos.dtype == torch.int64 and pos.numel() == 1 and T == 1 and ring.k.shape[0] >= B
        a.pos, a.chunk = pos.data_ptr(), ring.chunk
        a.k_ring, a.v_ring, a.ring_len = ring.k.data_ptr(), ring.v.data_ptr(), ring.len.data_ptr()
        a.ring_stride_b, a.ring_stride_g, a.ring_stride_s = ring.k.stride()[:3]
    check("socket_rope_half_rows", core().socket_rope_half_rows(ctypes.byref(a), stream_ptr(proj.device)))
    return (q, k) if pos is None else q


def _chunk_args(q: Tensor, ring, scale: float, softcap: float, G: int) -> ChunkAttention:
    B, T, H, D = q.shape
    assert q.stride(3) == 1
    return ChunkAttention(q=q.data_ptr(), q_stride_b=q.stride(0), q_stride_t=q.stride(1), q_stride_h=q.stride(2),
                          k_ring=ring.k.data_ptr(), v_ring=ring.v.data_ptr(), ring_stride_b=ring.k.stride(0),
                          ring_stride_g=ring.k.stride(1), ring_stride_s=ring.k.stride(2), dtype=dtype_enum(q.dtype),
                          B=B, T=T, H=H, G=G, D=D, chunk=ring.chunk, scale=scale, softcap=softcap)


@torch.no_grad()
def chunk_attend(q: Tensor, k: Tensor, v: Tensor, ring, pos0: int, scale: float, softcap: float,
                 force_simple: bool = False) -> Tensor:
    """Attention of a portion at pos0 inside its chunks: q [B,T,H,D], k / v [B,T,G,D] (any strides),
    older keys from `ring`, which then takes the portion's last chunk."""
    B, T, H, D = q.shape
    G = k.shape[2]
    out = torch.empty(B, T, H, D, dtype=q.dtype, device=q.device)
    a = _chunk_args(q, ring, scale, softcap, G)
    a.k_new, (a.k_stride_b, a.k_stride_t, a.k_stride_g) = k.data_ptr(), k.stride()[:3]
    a.v_new, (a.v_stride_b, a.v_stride_t, a.v_stride_g) = v.data_ptr(), v.stride()[:3]
    a.pos0, a.k_from, a.out, a.force_simple = pos0, pos0, out.data_ptr(), int(force_simple)
    L, s = core(), stream_ptr(q.device)
    check("socket_chunk_attend", L.socket_chunk_attend(ctypes.byref(a), s))
    check("socket_chunk_ring_store", L.socket_chunk_ring_store(
        ptr(k), *k.stride()[:3], ptr(v), *v.stride()[:3], ptr(ring.k), ptr(ring.v), *ring.k.stride()[:3],
        dtype_enum(q.dtype), B, T, G, D, ring.chunk, pos0, s))
    return out


@torch.no_grad()
def chunk_attend_step(q: Tensor, ring, pos: Tensor, G: int, scale: float, softcap: float) -> Tensor:
    """One token at the device position `pos`, whose key is in `ring` already: q [B,1,H,D]."""
    B, _, H, D = q.shape
    out = torch.empty(B, 1, H, D, dtype=q.dtype, device=q.device)
    if q.dtype == torch.bfloat16 and D % 8 == 0 and D <= 128 and H // G <= 16:
        # the ring's visible rows are a prefix: the split-K matrix-core kernel
        L, rows = core(), ring.k.shape[2]
        nbytes = L.socket_dense_decode_capped_workspace_bytes(B, H, rows)
        ws = torch.empty((nbytes + 3) // 4, dtype=torch.float32, device=q.device)
        check("socket_dense_decode_capped", L.socket_dense_decode_capped(
            ptr(q), ptr(ring.k), ptr(ring.v), dtype_enum(q.dtype), q.stride(0), q.stride(2), *ring.k.stride()[:3],
            *ring.v.stride()[:3], ptr(ring.len), ptr(out), out.stride(0), out.stride(2), ptr(ws), nbytes, B, H, G, D,
            rows, scale, softcap, stream_ptr(q.device)))
        return out
    a = _chunk_args(q, ring, scale, softcap, G)
    a.pos, a.out = pos.data_ptr(), out.data_ptr()
    check("socket_chunk_attend", core().socket_chunk_attend(ctypes.byref(a), stream_ptr(q.device)))
    return out


ENDLESS = 2 ** 31 - 1      # a chunk that no position leaves


@torch.no_grad()
def causal_attend(q: Tensor, k: Tensor, k_shared: Tensor, v: Tensor, pos0: int, scale: float, gate: Optional[Tensor] = None,
                  force_simple: bool = False) -> Tensor:
    """Causal attention of queries q [B,T,H,D+D2] at positions pos0 .. over the keys of every position:
    k [B,S,H,D] beside k_shared [B,S,D2] of all heads, values v [B,S,H,Dv], S = pos0 + T (any strides,
    last dimension contiguous).  Times sigmoid(gate), gate [B,T,H*Dv]; returns [B,T,H,Dv]."""
    B, T, H, dq = q.shape
    D, D2, dv = k.shape[3], k_shared.shape[2], v.shape[3]
    assert dq == D + D2 and k.shape[1] == v.shape[1] == k_shared.shape[1] == pos0 + T and k.shape[2] == v.shape[2] == H
    assert all(t.stride(-1) == 1 and t.dtype == q.dtype for t in (q, k, k_shared, v) + (() if gate is None else (gate,)))
    out = torch.empty(B, T, H, dv, dtype=q.dtype, device=q.device)
    a = ChunkAttention(q=q.data_ptr(), q_stride_b=q.stride(0), q_stride_t=q.stride(1), q_stride_h=q.stride(2),
                       dtype=dtype_enum(q.dtype), B=B, T=T, H=H, G=H, D=D, D2=D2, Dv=dv, chunk=ENDLESS, pos0=pos0, k_from=0,
                       scale=scale, out=out.data_ptr(), force_simple=int(force_simple))
    a.k_new, (a.k_stride_b, a.k_stride_t, a.k_stride_g) = k.data_ptr(), k.stride()[:3]
    a.v_new, (a.v_stride_b, a.v_stride_t, a.v_stride_g) = v.data_ptr(), v.stride()[:3]
    a.k2, (a.k2_stride_b, a.k2_stride_t) = k_shared.data_ptr(), k_shared.stride()[:2]
    if gate is not None:
        assert gate.shape == (B, T, H * dv)
        a.gate, (a.gate_stride_b, a.gate_stride_t) = gate.data_ptr(), gate.stride()[:2]
    check("socket_chunk_attend", core().socket_chunk_attend(ctypes.byref(a), stream_ptr(q.device)))
    return out


def _latent_args(src: Optional[Tensor], cache, dim: int, H: int, B: int, T: int, cos_sin: Tensor, pos0: int,
                 pos: Optional[Tensor], eps: float) -> Latent:
    a = Latent(dtype=dtype_enum(cache.rows.dtype), B=B, T=T, H=H, dim=dim, rot=cache.rot, rank=cache.rank, eps=eps,
               cos_sin=cos_sin.data_ptr(), n_pos=min(cos_sin.shape[0], cache.rows.shape[1]), pos0=pos0,
               cache=cache.rows.data_ptr(), cache_stride_b=cache.rows.stride(0), cache_stride_t=cache.rows.stride(1))
    assert cos_sin.dtype == torch.float32 and cos_sin.is_contiguous() and cache.rows.shape[0] >= B
    if src is not None:
        assert src.stride(2) == 1 and src.dtype in (torch.float32, cache.rows.dtype)
        a.in_, a.in_f32 = src.data_ptr(), int(src.dtype == torch.float32)
        a.in_stride_b, a.in_stride_t = src.stride()[:2]
    else:
        a.in_f32 = int(cache.rows.dtype == torch.float32)
    if pos is not None:
        assert pos.dtype == torch.int64 and pos.numel() == 1 and T == 1
        a.pos = pos.data_ptr()
    return a


@torch.no_grad()
def latent_rows(proj: Tensor, cache, cq_off: int, q_rank: int, c_off: int, rot_off: int, q_norm: Tensor, c_norm: Tensor,
                eps: float, cos_sin: Tensor, *, pos0: int = 0, pos: Optional[Tensor] = None) -> Tensor:
    """Cache rows of the projected rows proj [B,T,N] (normed latent, rotated shared key part); returns
    the normed query latent [B,T,q_rank]."""
    B, T, _ = proj.shape
    a = _latent_args(proj, cache, 1, 1, B, T, cos_sin, pos0, pos, eps)
    cq = torch.empty(B, T, q_rank, dtype=cache.rows.dtype, device=proj.device)
    a.cq_off, a.q_rank, a.c_off, a.rot_off = cq_off, q_rank, c_off, rot_off
    a.q_norm, a.c_norm, a.cq_out = q_norm.data_ptr(), c_norm.data_ptr(), cq.data_ptr()
    check("socket_latent_rows", core().socket_latent_rows(ctypes.byref(a), stream_ptr(proj.device)))
    return cq


@torch.no_grad()
def rotate_tail(q: Tensor, rot: int, cos_sin: Tensor, pos0: int) -> Tensor:
    """Rotate-half of the last `rot` elements of every head of q [B,T,H,D], in place."""
    B, T, H, D = q.shape
    assert q.is_contiguous() and cos_sin.dtype == torch.float32 and cos_sin.is_contiguous()
    check("socket_rotate_tail", core().socket_rotate_tail(ptr(q), dtype_enum(q.dtype), B, T, H, D - rot, rot, ptr(cos_sin),
                                                          cos_sin.shape[0], pos0, stream_ptr(q.device)))
    return q


@torch.no_grad()
def latent_absorb(q: Tensor, w_uk: Tensor, cache, cos_sin: Tensor, *, pos0: int = 0, pos: Optional[Tensor] = None,
                  proj: Optional[Tensor] = None, c_off: int = 0, rot_off: int = 0, c_norm: Optional[Tensor] = None,
                  eps: float = 0.0) -> Tensor:
    """q fp32 [B,T,H,dim+rot] as projected -> queries over the cache rows [B,T,H,width].  With `proj`
    the new tokens' cache rows are written too."""
    B, T, H, dq = q.shape
    assert q.dtype == torch.float32 and q.is_contiguous() and w_uk.is_contiguous() and w_uk.dtype == cache.rows.dtype
    assert w_uk.shape == (H * (dq - cache.rot), cache.rank)
    a = _latent_args(proj, cache, dq - cache.rot, H, B, T, cos_sin, pos0, pos, eps)
    out = torch.empty(B, T, H, cache.width, dtype=cache.rows.dtype, device=q.device)
    a.q, a.w_uk, a.q_lat = q.data_ptr(), w_uk.data_ptr(), out.data_ptr()
    if proj is not None:
        a.append, a.c_off, a.rot_off, a.c_norm = 1, c_off, rot_off, c_norm.data_ptr()
    check("socket_latent_absorb", core().socket_latent_absorb(ctypes.byref(a), stream_ptr(q.device)))
    return out


def latent_splits(capacity: int, tokens: int, heads: int) -> int:
    """Workgroups that share a token's keys: a tile of 64 keys each, from 128 tiles on at least two, and
    about one workgroup per CU at most."""
    tiles = (capacity + 63) // 64
    return max(1, min(256 // (tokens * ((heads + 15) // 16)), tiles if tiles <= 128 else max(128, tiles // 2)))


@torch.no_grad()
def latent_attend(q_lat: Tensor, cache, scale: float, w_uv: Tensor, vdim: int, gate: Optional[Tensor] = None, *, pos0: int = 0,
                  pos: Optional[Tensor] = None, force_simple: bool = False) -> Tensor:
    """Queries q_lat [B,T,H,width] at pos0 .. (or the device position `pos`, T = 1) over the cache rows,
    the value product and the sigmoid gate [B,T,H*vdim] (fp32 or the model's dtype): [B,T,H*vdim]."""
    B, T, H, width = q_lat.shape
    assert q_lat.is_contiguous() and width == cache.width and w_uv.is_contiguous() and w_uv.shape == (H * vdim, cache.rank)
    rows, dt = cache.rows, cache.rows.dtype
    a = LatentAttend(dtype=dtype_enum(dt), B=B, T=T, H=H, rank=cache.rank, rot=cache.rot, vdim=vdim, q_lat=q_lat.data_ptr(),
                     cache=rows.data_ptr(), cache_stride_b=rows.stride(0), cache_stride_t=rows.stride(1), n_pos=rows.shape[1],
                     pos0=pos0, scale=scale, splits=1, w_uv=w_uv.data_ptr())
    if pos is not None:
        assert pos.dtype == torch.int64 and pos.numel() == 1 and T == 1
        a.pos = pos.data_ptr()
    L, s = core(), stream_ptr(rows.device)
    rank_p = (cache.rank + 7) // 8 * 8
    if dt == torch.bfloat16 and not force_simple and rank_p <= 512 and width <= 640:
        a.splits = latent_splits(rows.shape[1], B * T, H)
        o = torch.empty(B * T, a.splits, H, rank_p, dtype=torch.float32, device=rows.device)
        ml = torch.empty(B * T, a.splits, H, 2, dtype=torch.float32, device=rows.device)
        a.o, a.ml = o.data_ptr(), ml.data_ptr()
        check("socket_latent_attend", L.socket_latent_attend(ctypes.byref(a), s))
    else:
        raw = torch.empty(B, T, H, rank_p, dtype=dt, device=rows.device)
        c = ChunkAttention(q=q_lat.data_ptr(), q_stride_b=q_lat.stride(0), q_stride_t=q_lat.stride(1), q_stride_h=width,
                           dtype=dtype_enum(dt), B=B, T=T, H=H, G=1, D=width, Dv=rank_p, chunk=ENDLESS, pos0=pos0, k_from=0,
                           scale=scale, out=raw.data_ptr(), force_simple=1)
        c.k_new = c.v_new = c.k_ring = c.v_ring = rows.data_ptr()
        c.k_stride_b = c.v_stride_b = c.ring_stride_b = rows.stride(0)
        c.k_stride_t = c.v_stride_t = c.ring_stride_s = rows.stride(1)
        if pos is not None:
            c.pos = pos.data_ptr()
        check("socket_chunk_attend", L.socket_chunk_attend(ctypes.byref(c), s))
        o = raw.float()
        a.o = o.data_ptr()
    out = torch.empty(B, T, H * vdim, dtype=dt, device=rows.device)
    a.out = out.data_ptr()
    if gate is not None:
        assert gate.stride(2) == 1 and gate.shape == out.shape and gate.dtype in (torch.float32, dt)
        a.gate, a.gate_f32 = gate.data_ptr(), int(gate.dtype == torch.float32)
        a.gate_stride_b, a.gate_stride_t = gate.stride()[:2]
    check("socket_latent_values", L.socket_latent_values(ctypes.byref(a), s))
    return out


@torch.no_grad()
def tanh_rows(x: Tensor) -> Tensor:
    """tanh of the rows x [B,T,n], a slice of wider rows, as a contiguous tensor."""
    B, T, n = x.shape
    if x.stride(2) != 1 or (B > 1 and x.stride(0) != T * x.stride(1)):
        x = x.contiguous()
    y = torch.empty(B, T, n, dtype=x.dtype, device=x.device)
    check("socket_tanh_rows", core().socket_tanh_rows(ptr(x), x.stride(1), ptr(y), dtype_enum(x.dtype), B * T, n,
                                                      stream_ptr(x.device)))
    return y


SCAN_SEGMENT = 2048     # tokens per prep / scan launch: bounds the workspace


@torch.no_grad()
def recurrence_scan(a: Recurrence, proj: Tensor, decay_z: Tensor, gate_z: Optional[Tensor], pos0: int,
                    fresh: bool) -> Tensor:
    """A portion proj [B,T,N] at pos0 through the recurrence described by `a` (weights, offsets and
    state filled in); returns [B,T,H*dv] and leaves the state at the portion's end."""
    B, T, _ = proj.shape
    L, s = core(), stream_ptr(proj.device)
    out = torch.empty(B, T, a.H * a.dv, dtype=proj.dtype, device=proj.device)
    a.B, a.T = B, T
    a.proj, a.proj_stride_b, a.proj_stride_t = proj.data_ptr(), proj.stride(0), proj.stride(1)
    assert decay_z.is_contiguous() and (gate_z is None or gate_z.is_contiguous())
    a.decay_z, a.decay_z_f32 = decay_z.data_ptr(), int(decay_z.dtype == torch.float32)
    a.gate_z = None if gate_z is None else gate_z.data_ptr()
    a.pos, a.pos0, a.out = None, pos0, out.data_ptr()
    n_max = min(T, SCAN_SEGMENT)
    nbytes = L.socket_recurrence_workspace_bytes(B, n_max, a.H, a.dk, a.dv, a.rule)
    ws = torch.empty((nbytes + 3) // 4, dtype=torch.float32, device=proj.device)
    o_buf = torch.empty(B, n_max, a.H, a.dv, dtype=torch.float32, device=proj.device)
    a.workspace, a.workspace_bytes, a.o_buf = ws.data_ptr(), nbytes, o_buf.data_ptr()
    for t0 in range(0, T, n_max):
        a.t0, a.n, a.fresh = t0, min(n_max, T - t0), int(fresh and t0 == 0)
        check("socket_recurrence_scan", L.socket_recurrence_scan(ctypes.byref(a), s))
    a.fresh = int(fresh)
    check("socket_recurrence_conv_tail", L.socket_recurrence_conv_tail(ctypes.byref(a), s))
    return out


@torch.no_grad()
def recurrence_step(a: Recurrence, proj: Tensor, pos: Tensor) -> Tensor:
    """One token per sequence, proj [B,1,N] at the device position `pos`: [B,1,H*dv]."""
    B = proj.shape[0]
    out = torch.empty(B, 1, a.H * a.dv, dtype=proj.dtype, device=proj.device)
    assert pos.dtype == torch.int64 and pos.numel() == 1
    a.B, a.T, a.fresh = B, 1, 0
    a.proj, a.proj_stride_b, a.proj_stride_t = proj.data_ptr(), proj.stride(0), proj.stride(1)
    a.pos, a.out = pos.data_ptr(), out.data_ptr()
    check("socket_recurrence_step", core().socket_recurrence_step(ctypes.byref(a), stream_ptr(proj.device)))
    return out
