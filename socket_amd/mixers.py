"""Token mixers of decoders assembled from a list of layers: softmax attention inside
chunks of the position axis, attention over a latent row per token, and gated linear
recurrences with or without the delta rule, plain or generalized.  Each is a *branch* of a layer: it names the columns it wants of the layer's one
input projection, turns them into the concatenated head outputs, and owns the output
projection that follows.  Constants (scales, caps, chunk, taps, decay and gate forms,
rates) are parameters of the spec.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, Optional, Tuple

import torch
import torch.nn as nn
from torch import Tensor
from torch.nn import functional as F

from . import layer_ops
from ._lib import Recurrence, dtype_enum
from .sequence_state import ChunkRing, LatentCache, RecurrentState


@dataclass
class ChunkAttentionSpec:
    heads: int
    kv_heads: int
    dim: int
    chunk: int
    rot_dims: int
    rot_base: float
    scale: float
    softcap: float = 0.0          # 0: none
    # (the values are the keys before their rotation: there is no value projection)


@dataclass
class RecurrenceSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    decay_rank: int               # inner width of the decay's two-matrix projection
    delta: bool                   # delta rule (with a write strength beta per head) or plain outer-product writes
    taps: int = 0                 # short causal convolution + SiLU on q, k, v; 0: neither
    unit_qk: bool = False
    decay: str = "exp_softplus"   # "exp_softplus": exp(-exp(A) softplus(z)); "sigmoid_root": sigmoid(z)^(1/tau);
                                  # "exp_sigmoid": exp(-decay_rate sigmoid(z))
    tau: float = 1.0
    gate: str = "sigmoid"         # of a two-matrix projection (gate_rank > 0) or of a full one
    gate_rank: int = 0
    # Generalized delta rule: removal at a rate per key channel, sigmoid of a projection with a bias,
    # along the unit key; what is written takes the key as it is.  Removal and decay both act on
    # the state before the token.  Its decay is "exp_sigmoid", of a tanh between the two matrices.
    removal: bool = False
    decay_rate: float = 1.0
    q_scale: Optional[float] = None   # None: dim ** -0.5
    norm_per_head: bool = False   # the read-outs' norm weight is [heads * vdim] instead of [vdim]


@dataclass
class LatentAttentionSpec:
    heads: int
    dim: int                      # unrotated query / key dimensions of a head
    rot_dim: int                  # rotated ones, whose key part all heads share
    vdim: int
    q_rank: int
    kv_rank: int
    rot_base: float
    scale: float


class StepContext:
    """What the layers of one step share.  A portion has the host position `pos0` (0: the
    sequence starts here); a single-token decode step has the device position `pos`.  `past`: the
    embedding output and every layer's result, where a design averages over depth."""
    __slots__ = ("pos0", "pos", "rope", "past")

    def __init__(self, pos0: Optional[int], pos: Optional[Tensor], rope: Dict[Tuple[float, int], Tensor],
                 past: Optional[Tensor] = None):
        self.pos0, self.pos, self.rope, self.past = pos0, pos, rope, past


class ColumnMap:
    """Rows of a fused projection: segments in order, each starting at a multiple of 8."""

    def __init__(self):
        self.offset: Dict[str, int] = {}
        self.rows: Dict[str, int] = {}
        self.total = 0

    def add(self, name: str, rows: int) -> None:
        self.offset[name], self.rows[name] = self.total, rows
        self.total += (rows + 7) // 8 * 8


class ChunkAttention(nn.Module):
    F32_STEP = False

    def __init__(self, spec: ChunkAttentionSpec, width: int, columns: ColumnMap, tag: str):
        super().__init__()
        assert spec.heads % spec.kv_heads == 0 and spec.rot_dims <= spec.dim and spec.rot_dims % 2 == 0
        self.spec, self.tag, self.cols = spec, tag, columns
        columns.add(tag + ".q", spec.heads * spec.dim)
        columns.add(tag + ".k", spec.kv_heads * spec.dim)
        self.o = nn.Parameter(torch.empty(width, spec.heads * spec.dim), requires_grad=False)
        self.state: Optional[ChunkRing] = None

    def alloc_state(self, batch: int, max_seq_length: int, dtype, device) -> None:
        c = self.spec
        self.state = ChunkRing(batch, max_seq_length, c.kv_heads, c.dim, c.chunk, dtype, device)

    def rope_key(self):
        return self.spec.rot_base, self.spec.rot_dims

    def heads(self, proj: Tensor, ctx: StepContext) -> Tensor:
        c, off = self.spec, self.cols.offset
        B, T, _ = proj.shape
        q_off, k_off = off[self.tag + ".q"], off[self.tag + ".k"]
        table = ctx.rope[(c.rot_base, c.rot_dims)]
        if ctx.pos is not None:
            q = layer_ops.rope_half(proj, q_off, k_off, c.heads, c.kv_heads, c.dim, c.rot_dims, table, pos=ctx.pos,
                                    ring=self.state)
            out = layer_ops.chunk_attend_step(q, self.state, ctx.pos, c.kv_heads, c.scale, c.softcap)
        else:
            q, k = layer_ops.rope_half(proj, q_off, k_off, c.heads, c.kv_heads, c.dim, c.rot_dims, table, pos0=ctx.pos0)
            v = proj[..., k_off:k_off + c.kv_heads * c.dim].view(B, T, c.kv_heads, c.dim)
            out = layer_ops.chunk_attend(q, k, v, self.state, ctx.pos0, c.scale, c.softcap)
        return out.view(B, T, c.heads * c.dim)


class LatentAttention(nn.Module):
    """Keys and values are products of a normed latent row per token; only that row and the shared
    rotated key part are cached.  A long portion expands keys and values of all its positions; a
    decode step or a portion of at most FEW tokens attends over the cache rows themselves, with
    the key product taken on the query's side and the value product on the weighted sum.  The
    output is gated by the sigmoid of a projection."""
    FEW = 8
    F32_STEP = True                   # a decode step's projected row stays fp32
    FP32 = ("q_norm", "c_norm")

    def __init__(self, spec: LatentAttentionSpec, width: int, eps: float, columns: ColumnMap, tag: str):
        super().__init__()
        c = spec
        assert c.rot_dim % 2 == 0 and c.rot_dim > 0
        self.spec, self.tag, self.cols, self.eps = spec, tag, columns, eps
        columns.add(tag + ".cq", c.q_rank)
        columns.add(tag + ".c", c.kv_rank)
        columns.add(tag + ".rot", c.rot_dim)
        columns.add(tag + ".g", c.heads * c.vdim)

        def param(*shape):
            return nn.Parameter(torch.empty(*shape), requires_grad=False)

        self.q_norm, self.c_norm = param(c.q_rank), param(c.kv_rank)
        self.uq = param(c.heads * (c.dim + c.rot_dim), c.q_rank)
        self.ukv = param(c.heads * (c.dim + c.vdim), c.kv_rank)     # all heads' key rows, then all value rows
        self.o = param(width, c.heads * c.vdim)
        self.state: Optional[LatentCache] = None

    @property
    def uk(self) -> Tensor:
        return self.ukv[:self.spec.heads * self.spec.dim]

    @property
    def uv(self) -> Tensor:
        return self.ukv[self.spec.heads * self.spec.dim:]

    def alloc_state(self, batch: int, max_seq_length: int, dtype, device) -> None:
        self.state = LatentCache(batch, max_seq_length, self.spec.kv_rank, self.spec.rot_dim, dtype, device)

    def rope_key(self):
        return self.spec.rot_base, self.spec.rot_dim

    def heads(self, proj: Tensor, ctx: StepContext) -> Tensor:
        c, t, off = self.spec, self.tag, self.cols.offset
        B, T, _ = proj.shape
        dt, dq = self.uq.dtype, c.dim + c.rot_dim
        table = ctx.rope[self.rope_key()]
        at = dict(c_off=off[t + ".c"], rot_off=off[t + ".rot"], c_norm=self.c_norm, eps=self.eps)
        gate = proj[..., off[t + ".g"]:off[t + ".g"] + c.heads * c.vdim]
        if ctx.pos is not None:
            cq = proj[..., off[t + ".cq"]:off[t + ".cq"] + c.q_rank]
            _, q = layer_ops.norm_linear(cq, None, self.q_norm, self.eps, self.uq, f32_out=True)
            q_lat = layer_ops.latent_absorb(q.view(B, T, c.heads, dq), self.uk, self.state, table, pos=ctx.pos, proj=proj, **at)
            return layer_ops.latent_attend(q_lat, self.state, c.scale, self.uv, c.vdim, gate, pos=ctx.pos)
        cq = layer_ops.latent_rows(proj, self.state, off[t + ".cq"], c.q_rank, q_norm=self.q_norm, cos_sin=table, pos0=ctx.pos0, **at)
        if 0 < ctx.pos0 and T <= self.FEW:
            q = layer_ops.linear_f32(cq, self.uq).view(B, T, c.heads, dq)
            q_lat = layer_ops.latent_absorb(q, self.uk, self.state, table, pos0=ctx.pos0)
            return layer_ops.latent_attend(q_lat, self.state, c.scale, self.uv, c.vdim, gate, pos0=ctx.pos0)
        q = layer_ops.rotate_tail(F.linear(cq, self.uq).view(B, T, c.heads, dq), c.rot_dim, table, ctx.pos0)
        S = ctx.pos0 + T
        rows = self.state.rows[:B, :S]
        kv = F.linear(rows[..., :c.kv_rank].reshape(B * S, c.kv_rank), self.ukv).view(B, S, c.heads * (c.dim + c.vdim))
        k, v = kv.split([c.heads * c.dim, c.heads * c.vdim], -1)
        k_rot = rows[..., self.state.rot_at:self.state.rot_at + c.rot_dim]
        out = layer_ops.causal_attend(q, k.unflatten(-1, (c.heads, c.dim)), k_rot, v.unflatten(-1, (c.heads, c.vdim)), ctx.pos0,
                                      c.scale, gate)
        return out.view(B, T, c.heads * c.vdim)


class GatedRecurrence(nn.Module):
    F32_STEP = False

    def __init__(self, spec: RecurrenceSpec, width: int, eps: float, columns: ColumnMap, tag: str):
        super().__init__()
        c = spec
        assert c.heads % c.kv_heads == 0
        self.spec, self.tag, self.cols, self.eps = spec, tag, columns, eps
        columns.add(tag + ".q", c.kv_heads * c.dim)
        columns.add(tag + ".k", c.kv_heads * c.dim)
        columns.add(tag + ".v", c.heads * c.vdim)
        columns.add(tag + ".a1", c.decay_rank)
        columns.add(tag + ".g", c.gate_rank or c.heads * c.vdim)
        if c.removal:
            assert c.delta and c.heads == c.kv_heads and not c.taps and not c.gate_rank and c.decay == "exp_sigmoid"
            columns.add(tag + ".rate", c.heads * c.dim)
        elif c.delta:
            columns.add(tag + ".b", c.heads)
        self.conv_channels = 2 * c.kv_heads * c.dim + c.heads * c.vdim

        def param(*shape):
            return nn.Parameter(torch.empty(*shape), requires_grad=False)

        self.o = param(width, c.heads * c.vdim)
        self.decay_w = param(c.heads * c.dim, c.decay_rank)
        self.gate_w = param(c.heads * c.vdim, c.gate_rank) if c.gate_rank else None
        # (fp32 whatever the model's dtype: what enters the recurrence is 32-bit)
        self.a_log = param(c.heads) if c.decay == "exp_softplus" else None
        self.decay_bias = param(c.heads * c.dim)
        self.rate_bias = param(c.heads * c.dim) if c.removal else None
        self.norm = param(c.heads * c.vdim if c.norm_per_head else c.vdim)
        self.conv_w = param(c.taps, self.conv_channels) if c.taps else None
        self.state: Optional[RecurrentState] = None

    FP32 = ("a_log", "decay_bias", "rate_bias", "norm", "conv_w")

    def rope_key(self):
        return None

    def alloc_state(self, batch: int, max_seq_length: int, dtype, device) -> None:
        c = self.spec
        self.state = RecurrentState(batch, c.heads, c.dim, c.vdim, c.taps - 1, self.conv_channels, dtype, device)

    def _args(self, dtype) -> Recurrence:
        c, off, t = self.spec, self.cols.offset, self.tag
        a = Recurrence(dtype=dtype_enum(dtype), H=c.heads, Hk=c.kv_heads, dk=c.dim, dv=c.vdim,
                       q_off=off[t + ".q"], k_off=off[t + ".k"], v_off=off[t + ".v"],
                       beta_off=off[t + ".b"] if c.delta and not c.removal else -1, decay_off=off[t + ".a1"], gate_off=off[t + ".g"],
                       taps=c.taps, unit_qk=int(c.unit_qk), q_scale=c.dim ** -0.5 if c.q_scale is None else c.q_scale,
                       decay_kind={"exp_softplus": 0, "sigmoid_root": 1, "exp_sigmoid": 2}[c.decay], decay_bias=self.decay_bias.data_ptr(),
                       inv_tau=1.0 / c.tau, decay_w=self.decay_w.data_ptr(), decay_rank=c.decay_rank,
                       gate_kind={"sigmoid": 0, "silu": 1}[c.gate], gate_rank=c.gate_rank,
                       norm_w=self.norm.data_ptr(), eps=self.eps, state=self.state.s.data_ptr())
        a.norm_per_head = int(c.norm_per_head)
        if c.removal:
            a.rule, a.rate_off, a.rate_bias = 1, off[t + ".rate"], self.rate_bias.data_ptr()
            a.decay_tanh, a.decay_rate = 1, c.decay_rate
        if self.a_log is not None:
            a.a_log = self.a_log.data_ptr()
        if self.gate_w is not None:
            a.gate_w = self.gate_w.data_ptr()
        if self.conv_w is not None:
            a.conv_w, a.conv_state = self.conv_w.data_ptr(), self.state.conv.data_ptr() or None
        return a

    def heads(self, proj: Tensor, ctx: StepContext) -> Tensor:
        c, off, t = self.spec, self.cols.offset, self.tag
        assert self.state.s.shape[0] == proj.shape[0], "the state holds another number of sequences"
        a = self._args(proj.dtype)
        if ctx.pos is not None:
            return layer_ops.recurrence_step(a, proj, ctx.pos)
        low = proj[..., off[t + ".a1"]:off[t + ".a1"] + c.decay_rank]
        z = layer_ops.linear_f32(layer_ops.tanh_rows(low) if c.removal else low, self.decay_w)
        gate = None
        if self.gate_w is not None:
            gate = F.linear(proj[..., off[t + ".g"]:off[t + ".g"] + c.gate_rank], self.gate_w)
        return layer_ops.recurrence_scan(a, proj, z, gate, ctx.pos0, fresh=ctx.pos0 == 0)
