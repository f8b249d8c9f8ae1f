"""The Guselix design: its config.json and its tensor names.

A layer's mixer is 'general_delta' (generalized delta rule) or 'latent_attention'; the
feed-forward is a gated SiLU unit with biases or absent.  A layer's result is averaged with the
results before it and the embedding output; the output matrix is the embedding table.  The
inner width of the decay's two matrices is not in the config; it is read from the tensors'
shapes.
"""
from __future__ import annotations

import math
from typing import Dict, Tuple

import torch

from .checkpoint import only, put
from .hybrid import BranchSpec, HybridArgs, HybridTransformer, LayerSpec, SiluGLUSpec
from .mixers import LatentAttention, LatentAttentionSpec, RecurrenceSpec

ARCHITECTURE = "Guselix"
DECAY_RATE = math.exp(-0.5)       # decays lie between exp(-DECAY_RATE) and 1


def general_delta(heads: int, dim: int, decay_rank: int) -> RecurrenceSpec:
    return RecurrenceSpec(heads=heads, kv_heads=heads, dim=dim, vdim=dim, decay_rank=decay_rank, delta=True, removal=True,
                          decay="exp_sigmoid", decay_rate=DECAY_RATE, q_scale=1.0, norm_per_head=True, gate="sigmoid")


def _latent(c: dict, where: str) -> LatentAttentionSpec:
    only(c, "heads dim rot_dim vdim q_rank kv_rank rot scale", where)
    only(c["rot"], "base dims", where + ".rot")
    if c["rot"]["dims"] != c["rot_dim"]:
        raise ValueError(f"config, {where}: rot.dims must equal rot_dim")
    return LatentAttentionSpec(heads=c["heads"], dim=c["dim"], rot_dim=c["rot_dim"], vdim=c["vdim"], q_rank=c["q_rank"],
                               kv_rank=c["kv_rank"], rot_base=float(c["rot"]["base"]), scale=float(c["scale"]))


def args_from_config(config: dict, shapes: Dict[str, Tuple[int, ...]]) -> HybridArgs:
    """`shapes`: tensor name -> shape, for the inner widths."""
    only(config, "architecture embedding layers norm vocab width", "top level")
    only(config["embedding"], "scale", "embedding")
    only(config["norm"], "eps", "norm")
    layers = []
    for i, lay in enumerate(config["layers"]):
        where = f"layer {i}"
        only(lay, "type mixer mlp", where)
        c = lay["mixer"]
        if lay["type"] == "general_delta":
            only(c, "heads dim", where)
            if f"l{i}.mix.w1" not in shapes:
                raise ValueError(f"the checkpoint has no tensor l{i}.mix.w1")
            spec = general_delta(c["heads"], c["dim"], shapes[f"l{i}.mix.w1"][0])
        elif lay["type"] == "latent_attention":
            spec = _latent(c, where)
        else:
            raise ValueError(f"config, {where}: unknown layer type {lay['type']!r}")
        mlp = None
        if lay["mlp"] is not None:
            only(lay["mlp"], "ff kind", where + ".mlp")
            if lay["mlp"]["kind"] != "dense":
                raise ValueError(f"config, {where}: unknown feed-forward kind {lay['mlp']['kind']!r}")
            mlp = SiluGLUSpec(lay["mlp"]["ff"], bias=True)
        layers.append(LayerSpec([BranchSpec(spec)], mlp))
    return HybridArgs(vocab_size=config["vocab"], dim=config["width"], layers=layers, norm_eps=float(config["norm"]["eps"]),
                      architecture=ARCHITECTURE, embed_scale=float(config["embedding"]["scale"]), tied_head=True,
                      post_norm=False, depth_average=True)


@torch.no_grad()
def load_tensors(model: HybridTransformer, take, ignore=lambda name: None) -> None:
    """Fill the model's parameters; `take(name)` hands over the checkpoint's tensor of that name,
    `ignore(name)` says that one is not needed."""
    put(model.tok_embeddings.weight, take("embed"), "embed")
    put(model.norm, take("final.norm"), "final.norm")
    for i, layer in enumerate(model.layers):
        pre = f"l{i}."
        mix = pre + "mix"
        layer.in_proj.zero_()
        br = layer.branches[0]

        def rows(name, src, tensor=None):
            at, n = layer.columns.offset[br.tag + "." + name], layer.columns.rows[br.tag + "." + name]
            put(layer.in_proj[at:at + n], take(src) if tensor is None else tensor, src)

        put(layer.norm1, take(pre + "norm1"), pre + "norm1")
        put(layer.dwa, take(pre + "dwa"), pre + "dwa")
        put(br.o, take(mix + ".o"), mix + ".o")
        rows("g", mix + ".g")
        c = br.spec
        if isinstance(br, LatentAttention):
            rows("cq", mix + ".dq")
            down = take(mix + ".dkv")
            if down.shape[0] != c.kv_rank + c.rot_dim:
                raise ValueError(f"tensor {mix}.dkv has shape {tuple(down.shape)}, expected {c.kv_rank + c.rot_dim} rows")
            rows("c", mix + ".dkv", down[:c.kv_rank])
            rows("rot", mix + ".dkv", down[c.kv_rank:])
            for dst, src in ((br.q_norm, ".dq.norm"), (br.c_norm, ".dkv.norm"), (br.uq, ".uq"), (br.uk, ".uk"), (br.uv, ".uv")):
                put(dst, take(mix + src), mix + src)
        else:
            for name, src in (("q", ".r"), ("k", ".k"), ("v", ".v"), ("a1", ".w1"), ("rate", ".a")):
                rows(name, mix + src)
            for dst, src in ((br.decay_w, ".w2"), (br.decay_bias, ".w0"), (br.rate_bias, ".a.b"), (br.norm, ".norm")):
                put(dst, take(mix + src), mix + src)
        if layer.spec.mlp is None:
            ignore(pre + "norm2")
        else:
            ff = layer.spec.mlp.ff
            put(layer.norm2, take(pre + "norm2"), pre + "norm2")
            for at, name in ((0, "gate"), (ff, "up")):
                put(layer.gate_up[at:at + ff], take(f"{pre}mlp.{name}"), f"{pre}mlp.{name}")
                put(layer.gate_up_bias[at:at + ff], take(f"{pre}mlp.{name}.b"), f"{pre}mlp.{name}.b")
            put(layer.down, take(pre + "mlp.down"), pre + "mlp.down")
            put(layer.down_bias, take(pre + "mlp.down.b"), pre + "mlp.down.b")
