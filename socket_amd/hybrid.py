"""Decoders given as a list of layers with different token mixers: the model class that
runs them through the framework's step functions.

`HybridTransformer` is driven like `model.Transformer` (setup_caches, forward with
input_pos / pos0 / last_only; generate.py's prefill, DecodeGraph and generate): a
portion of any length at a host position, or one token at a device position.  What a
sequence keeps between steps is sequence_state's; the residual stream is fp32.

A layer is one projection of the normalised stream for all of its branches, the
branches' heads (mixers.py), their output projections, and a gated feed-forward; a
design may normalise every sublayer's output again before it is added (post_norm), and may
average a layer's result with those before it and the embedding (depth_average).  Norm,
residual add, average and the norm after it are one launch (layer_ops.residual_norm).  In a
decode step the norm rides inside the product it feeds, and without a second norm the add
and the average inside the output product before it.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import List, Optional, Sequence, Tuple, Union

import torch
import torch.nn as nn
from torch import Tensor
from torch.nn import functional as F

from . import layer_ops
from .layer_ops import Depth, Pending
from .mixers import (ChunkAttention, ChunkAttentionSpec, ColumnMap, GatedRecurrence, LatentAttention, LatentAttentionSpec,
                     RecurrenceSpec, StepContext)
from .model import Transformer, precompute_freqs_cis


@dataclass
class ClampedGLUSpec:
    ff: int
    limit: float
    act = "clamped"
    bias = False


@dataclass
class SiluGLUSpec:
    ff: int
    bias: bool = False        # on all three projections
    act = "silu"
    limit = 0.0


@dataclass
class BranchSpec:
    spec: Union[ChunkAttentionSpec, LatentAttentionSpec, RecurrenceSpec]
    scale: float = 1.0
    name: str = ""            # its tensors' name inside the layer's mixer ("" for an only branch)


@dataclass
class LayerSpec:
    branches: List[BranchSpec]
    mlp: Optional[Union[ClampedGLUSpec, SiluGLUSpec]]


@dataclass
class HybridArgs:
    vocab_size: int
    dim: int
    layers: List[LayerSpec] = field(default_factory=list)
    norm_eps: float = 1e-5
    block_size: int = 1 << 20         # longest sequence generate() accepts
    architecture: str = ""
    embed_scale: float = 1.0          # of the looked-up rows
    tied_head: bool = False           # the output matrix is the embedding table
    post_norm: bool = True            # a second norm on every sublayer's output
    depth_average: bool = False       # a layer's result, all earlier ones and the embedding output, weighted

    @property
    def n_layer(self) -> int:
        return len(self.layers)


def _param(*shape) -> nn.Parameter:
    return nn.Parameter(torch.empty(*shape), requires_grad=False)


class HybridBlock(nn.Module):
    def __init__(self, cfg: HybridArgs, spec: LayerSpec, index: int):
        super().__init__()
        assert 1 <= len(spec.branches) <= 2
        self.spec, self.eps, self.index, self.embed_scale = spec, cfg.norm_eps, index, cfg.embed_scale
        self.columns = ColumnMap()
        self.branches = nn.ModuleList()
        for i, b in enumerate(spec.branches):
            tag = b.name or str(i)
            if isinstance(b.spec, ChunkAttentionSpec):
                self.branches.append(ChunkAttention(b.spec, cfg.dim, self.columns, tag))
            elif isinstance(b.spec, LatentAttentionSpec):
                self.branches.append(LatentAttention(b.spec, cfg.dim, cfg.norm_eps, self.columns, tag))
            else:
                self.branches.append(GatedRecurrence(b.spec, cfg.dim, cfg.norm_eps, self.columns, tag))
        self.in_proj = _param(self.columns.total, cfg.dim)
        self.norm1 = _param(cfg.dim)
        self.norm1b = _param(cfg.dim) if cfg.post_norm else None
        self.norm2b = self.gate_up_bias = self.down_bias = None
        if spec.mlp is not None:
            self.norm2 = _param(cfg.dim)
            self.norm2b = _param(cfg.dim) if cfg.post_norm else None
            self.gate_up = _param(2 * spec.mlp.ff, cfg.dim)
            self.down = _param(cfg.dim, spec.mlp.ff)
            if spec.mlp.bias:
                self.gate_up_bias, self.down_bias = _param(2 * spec.mlp.ff), _param(cfg.dim)
        self.dwa = _param(index + 2) if cfg.depth_average else None
        self.f32_step = any(br.F32_STEP for br in self.branches)

    FP32 = ("norm1", "norm1b", "norm2", "norm2b", "dwa")

    def _mix_out(self, proj: Tensor, ctx: StepContext, x: Tensor, depth: Optional[Depth]):
        """(x, pending) after the mixer; `depth`: this is the layer's last sublayer."""
        terms = [(br.heads(proj, ctx), br.o, b.scale) for br, b in zip(self.branches, self.spec.branches)]
        if depth is not None and ctx.pos is not None and self.norm1b is None and len(terms) == 1 and terms[0][2] == 1.0:
            return layer_ops.linear_residual(terms[0][0], terms[0][1], x, depth=depth)
        out = layer_ops.linear_terms(terms)
        out.post_w, out.depth = self.norm1b, depth
        return x, out

    def run(self, x: Optional[Tensor], pending: Optional[Pending], ctx: StepContext, dtype, embed=None, ids=None):
        """(x, pending) -> (x, pending): the stream without the last sublayer's output, and that output
        (None: it is in the stream)."""
        mlp = self.spec.mlp
        depth = None if self.dwa is None else Depth(ctx.past, self.index + 1, self.dwa)
        start = dict(embed=embed, ids=ids, embed_scale=self.embed_scale)
        if embed is not None and ctx.past is not None:
            start["x_out"] = ctx.past[0]
        if ctx.pos is not None:
            x, proj = layer_ops.norm_linear(x, pending, self.norm1, self.eps, self.in_proj, f32_out=self.f32_step, **start)
            x, pending = self._mix_out(proj, ctx, x, depth if mlp is None else None)
            if mlp is not None:
                gb, ub = (None, None) if self.gate_up_bias is None else self.gate_up_bias.split(mlp.ff)
                x, g = layer_ops.norm_linear(x, pending, self.norm2, self.eps, self.gate_up[:mlp.ff],
                                             up_weight=self.gate_up[mlp.ff:], act=mlp.act, limit=mlp.limit, bias=gb, up_bias=ub)
                if self.norm2b is None:
                    return layer_ops.linear_residual(g, self.down, x, self.down_bias, depth)
                assert self.down_bias is None
                pending = layer_ops.linear_terms([(g, self.down, 1.0)])
                pending.post_w, pending.depth = self.norm2b, depth
            return x, pending
        x, h = layer_ops.residual_norm(x, pending, self.norm1, self.eps, dtype, **start)
        x, pending = self._mix_out(F.linear(h, self.in_proj), ctx, x, depth if mlp is None else None)
        if mlp is not None:
            x, h = layer_ops.residual_norm(x, pending, self.norm2, self.eps, dtype)
            g = layer_ops.gated_unit(F.linear(h, self.gate_up, self.gate_up_bias), mlp.act, mlp.limit)
            pending = Pending(F.linear(g, self.down, self.down_bias), post_w=self.norm2b, depth=depth)
        return x, pending


class HybridTransformer(Transformer):
    def __init__(self, config: HybridArgs) -> None:
        nn.Module.__init__(self)
        self.config = config
        self.tok_embeddings = nn.Embedding(config.vocab_size, config.dim)
        self.layers = nn.ModuleList(HybridBlock(config, spec, i) for i, spec in enumerate(config.layers))
        self.norm = _param(config.dim)
        self.output = None if config.tied_head else nn.Linear(config.dim, config.vocab_size, bias=False)
        self.requires_grad_(False)
        self.max_batch_size = -1
        self.max_seq_length = -1
        self.rope = {}
        self._filled: Optional[int] = None        # positions fed so far, while the host knows

    FP32 = ("norm",)

    def cast(self, device, dtype) -> "HybridTransformer":
        """Parameters to `device`, matrices in `dtype` and the vectors of norms and recurrences in fp32."""
        for m in self.modules():
            keep = getattr(m, "FP32", ())
            for name, p in list(m._parameters.items()):
                if p is not None:
                    p.data = p.data.to(device=device, dtype=torch.float32 if name in keep else dtype)
        return self

    # ---- state ------------------------------------------------------------------------
    def setup_caches(self, max_batch_size, max_seq_length):
        if self.max_seq_length >= max_seq_length and self.max_batch_size == max_batch_size:
            return
        w = self.tok_embeddings.weight
        max_seq_length = max(self.max_seq_length, max_seq_length)
        self.max_batch_size, self.max_seq_length = max_batch_size, max_seq_length
        self.rope = {}
        for layer in self.layers:
            for br in layer.branches:
                br.alloc_state(max_batch_size, max_seq_length, w.dtype, w.device)
                key = br.rope_key()
                if key is not None and key not in self.rope:
                    self.rope[key] = precompute_freqs_cis(max_seq_length, key[1], key[0],
                                                          dtype=torch.float32).to(w.device)
        self._filled = None

    def step_state(self) -> List[Tensor]:
        return [t for layer in self.layers for br in layer.branches for t in br.state.overwritten_by_a_step()]

    # ---- the step -----------------------------------------------------------------------
    def _positions(self, idx: Tensor, input_pos: Tensor, pos0: Optional[int]):
        assert self.max_seq_length > 0, "Caches must be initialized first"
        input_pos, pos0 = self._check_positions(idx, input_pos, pos0)
        if idx.shape[0] != self.max_batch_size:
            raise RuntimeError(f"the caches hold {self.max_batch_size} sequences, the step brings {idx.shape[0]}")
        if pos0 is None:
            self._filled = None
        else:
            if pos0 > 0 and self._filled is not None and pos0 != self._filled:
                raise RuntimeError(f"a portion at position {pos0} does not continue the {self._filled} tokens fed so far")
            self._filled = pos0 + idx.shape[1]
        return input_pos, pos0

    def _run(self, idx: Tensor, input_pos: Tensor, sparse: bool, pos0: Optional[int], last_only: bool,
             rows: Optional[Sequence[int]] = None, collect: Optional[list] = None) -> Tensor:
        if sparse:
            raise ValueError("this model has no sparse attention path (decode_type must be 'dense')")
        input_pos, pos0 = self._positions(idx, input_pos, pos0)
        ids = idx.contiguous()
        w = self.tok_embeddings.weight
        past = None
        if self.config.depth_average:
            past = torch.empty(len(self.layers) + 1, *ids.shape, self.config.dim, dtype=torch.float32, device=w.device)
        ctx = StepContext(pos0, input_pos if pos0 is None else None, self.rope, past)
        head = w if self.output is None else self.output.weight
        eps = self.config.norm_eps
        x: Optional[Tensor] = None
        pending: Optional[Pending] = None
        embed, tok = w, ids
        for layer in self.layers:
            x, pending = layer.run(x, pending, ctx, w.dtype, embed=embed, ids=tok)
            embed = tok = None
            if collect is not None:
                collect.append(layer_ops.residual_norm(x, pending, self.norm, eps, w.dtype)[0])
        if ctx.pos is not None:
            return layer_ops.norm_linear(x, pending, self.norm, eps, head, f32_out=True)[1]
        _, h = layer_ops.residual_norm(x, pending, self.norm, eps, w.dtype)
        if rows is not None:
            h = h[:, list(rows)]
        elif last_only:
            h = h[:, -1:]
        return layer_ops.linear_f32(h.contiguous(), head)
