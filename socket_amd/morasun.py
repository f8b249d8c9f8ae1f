"""The Morasun design: its config.json and its tensor names.

A layer is 'parallel' (softcapped attention inside chunks beside a gated delta rule,
both on the same input, added with two scales) or 'gla' (gated linear attention); the
feed-forward is a clamped gated unit or absent.  The inner widths of the two-matrix
projections are not in the config; they are read from the tensors' shapes.
"""
from __future__ import annotations

from typing import Dict, Tuple

import torch

from .checkpoint import only, put
from .hybrid import BranchSpec, ClampedGLUSpec, HybridArgs, HybridTransformer, LayerSpec
from .mixers import ChunkAttention, ChunkAttentionSpec, RecurrenceSpec

ARCHITECTURE = "Morasun"


def _attention(c: dict, where: str) -> ChunkAttentionSpec:
    only(c, "heads kv_heads dim vdim mask rot scale softcap", where)
    only(c["mask"], "size", where + ".mask")
    only(c["rot"], "base dims", where + ".rot")
    if c["vdim"] != c["dim"]:
        raise ValueError(f"config, {where}: the values are the keys, so vdim must equal dim")
    return ChunkAttentionSpec(heads=c["heads"], kv_heads=c["kv_heads"], dim=c["dim"], chunk=c["mask"]["size"],
                              rot_dims=c["rot"]["dims"], rot_base=float(c["rot"]["base"]), scale=float(c["scale"]),
                              softcap=float(c["softcap"]))


def _delta(c: dict, ranks: Tuple[int, int], where: str) -> RecurrenceSpec:
    only(c, "heads kv_heads dim vdim conv", where)
    return RecurrenceSpec(heads=c["heads"], kv_heads=c["kv_heads"], dim=c["dim"], vdim=c["vdim"], decay_rank=ranks[0],
                          delta=True, taps=c["conv"], unit_qk=True, decay="exp_softplus", gate="sigmoid",
                          gate_rank=ranks[1])


def _gla(c: dict, rank: int, where: str) -> RecurrenceSpec:
    only(c, "heads dim vdim tau", where)
    return RecurrenceSpec(heads=c["heads"], kv_heads=c["heads"], dim=c["dim"], vdim=c["vdim"], decay_rank=rank,
                          delta=False, decay="sigmoid_root", tau=float(c["tau"]), gate="silu")


def args_from_config(config: dict, shapes: Dict[str, Tuple[int, ...]]) -> HybridArgs:
    """`shapes`: tensor name -> shape, for the inner widths."""
    only(config, "architecture layers norm vocab width", "top level")
    only(config["norm"], "eps", "norm")
    layers = []
    for i, lay in enumerate(config["layers"]):
        where, pre = f"layer {i}", f"l{i}.mix"
        only(lay, "type mixer mlp", where)
        c = lay["mixer"]
        if lay["type"] == "parallel":
            only(c, "left right left_scale right_scale", where)
            ranks = (shapes[pre + ".right.a1"][0], shapes[pre + ".right.g1"][0])
            branches = [BranchSpec(_attention(c["left"], where + ".left"), float(c["left_scale"]), "left"),
                        BranchSpec(_delta(c["right"], ranks, where + ".right"), float(c["right_scale"]), "right")]
        elif lay["type"] == "gla":
            branches = [BranchSpec(_gla(c, shapes[pre + ".a1"][0], where))]
        else:
            raise ValueError(f"config, {where}: unknown layer type {lay['type']!r}")
        mlp = None
        if lay["mlp"] is not None:
            only(lay["mlp"], "ff kind limit", where + ".mlp")
            if lay["mlp"]["kind"] != "dense":
                raise ValueError(f"config, {where}: unknown feed-forward kind {lay['mlp']['kind']!r}")
            mlp = ClampedGLUSpec(lay["mlp"]["ff"], float(lay["mlp"]["limit"]))
        layers.append(LayerSpec(branches, mlp))
    return HybridArgs(vocab_size=config["vocab"], dim=config["width"], layers=layers, norm_eps=float(config["norm"]["eps"]),
                      architecture=ARCHITECTURE)


@torch.no_grad()
def load_tensors(model: HybridTransformer, take, ignore=lambda name: None) -> None:
    """Fill the model's parameters; `take(name)` hands over the checkpoint's tensor of that name,
    `ignore(name)` says that one is not needed."""
    put(model.tok_embeddings.weight, take("embed"), "embed")
    put(model.norm, take("final.norm"), "final.norm")
    put(model.output.weight, take("head"), "head")
    for i, layer in enumerate(model.layers):
        pre = f"l{i}."
        layer.in_proj.zero_()

        def rows(tag, name, src):
            at, n = layer.columns.offset[tag + "." + name], layer.columns.rows[tag + "." + name]
            put(layer.in_proj[at:at + n], take(src), src)

        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if layer.spec.mlp is not None else ()):
            put(getattr(layer, n), take(pre + n), pre + n)
        for br, b in zip(layer.branches, layer.spec.branches):
            mix = pre + "mix" + ("." + b.name if b.name else "")
            t, c = br.tag, b.spec
            put(br.o, take(mix + ".o"), mix + ".o")
            rows(t, "q", mix + ".q")
            rows(t, "k", mix + ".k")
            if isinstance(br, ChunkAttention):
                continue
            rows(t, "v", mix + ".v")
            rows(t, "a1", mix + ".a1")
            put(br.decay_w, take(mix + ".a2"), mix + ".a2")
            put(br.norm, take(mix + ".norm"), mix + ".norm")
            if c.delta:
                rows(t, "b", mix + ".b")
                rows(t, "g", mix + ".g1")
                put(br.gate_w, take(mix + ".g2"), mix + ".g2")
                put(br.a_log, take(mix + ".A_log"), mix + ".A_log")
                put(br.decay_bias, take(mix + ".dt_bias"), mix + ".dt_bias")
            else:
                rows(t, "g", mix + ".g")
                put(br.decay_bias, take(mix + ".a2.b"), mix + ".a2.b")
            if c.delta:
                at = 0
                for n in ("q", "k", "v"):
                    w = take(f"{mix}.{n}.conv")
                    if w.shape[1] != c.taps:
                        raise ValueError(f"tensor {mix}.{n}.conv has {w.shape[1]} taps, the config says {c.taps}")
                    put(br.conv_w[:, at:at + w.shape[0]], w.t(), f"{mix}.{n}.conv")
                    at += w.shape[0]
        if layer.spec.mlp is None:
            ignore(pre + "norm2")
            ignore(pre + "norm2b")
        else:
            ff = layer.spec.mlp.ff
            put(layer.gate_up[:ff], take(pre + "mlp.gate"), pre + "mlp.gate")
            put(layer.gate_up[ff:], take(pre + "mlp.up"), pre + "mlp.up")
            put(layer.down, take(pre + "mlp.down"), pre + "mlp.down")
