"""The Guselix design on the device against the plain restatement in
oracle/guselix_oracle.py: each mechanism alone, then whole models in portions, token by
token, in batches, in reused state, and through generate() and bin/trace_run."""
import json
import os
import random
import subprocess
import sys

import numpy as np
import pytest
import torch

from oracle import guselix_oracle as go
from oracle import hybrid_oracle as ho
from tests import guselix_models as gm
from tests import hybrid_models as hm
from tests.test_hybrid_gpu import _feed, _rand

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
F32, BF16 = torch.float32, torch.bfloat16
TOL = {F32: 3e-5, BF16: 1e-1}       # of the worst token
MEAN_TOL = {F32: 1.5e-5, BF16: 3e-2}


def _row_error(got, want):
    """Largest error of a row relative to that row (rows far below the rest: to a tenth of the rest)."""
    got, want = got.double(), want.double()
    size = want.pow(2).mean(-1).sqrt()
    return float(((got - want).pow(2).mean(-1).sqrt() / size.clamp(min=0.1 * float(want.pow(2).mean().sqrt()))).max())


# ---- rows: embedding scale, average over depth, gated unit, biases ---------------------------------

@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("rows,dim,n", [(1, 40, 1), (5, 37, 3), (3, 2056, 9), (2, 4096, 70)])
def test_residual_norm_with_average_over_depth(dev, dtype, rows, dim, n):
    from socket_amd import layer_ops
    g = torch.Generator().manual_seed(dim)
    x, a, w, dwa = _rand(g, rows, dim), _rand(g, rows, dim), 1 + 0.2 * _rand(g, dim), _rand(g, n + 1)
    past = _rand(g, n + 2, rows, dim)
    res = x + 0.7 * a
    want = go.depth_average(list(past[:n]) + [res], dwa)
    p = past.to(dev, F32)
    before = p.clone()
    depth = layer_ops.Depth(p, n, dwa.to(dev, F32))
    gx, gh = layer_ops.residual_norm(x.to(dev, F32), layer_ops.Pending(a.to(dev, dtype), 0.7, depth=depth), w.to(dev, F32), 1e-4, dtype)
    assert hm.rms_error(gx.cpu(), want) < 1e-6
    assert hm.rms_error(gh.cpu(), ho.rms_norm(want, 1e-4, w)) < (1e-6 if dtype == F32 else 3e-3)
    assert hm.rms_error(p[n].cpu(), res) < 1e-6                  # the result itself is what later layers average
    assert torch.equal(p[:n], before[:n]) and torch.equal(p[n + 1:], before[n + 1:])
    # the scaled embedding as the stream's start, kept where it is told to
    table = _rand(g, 11, dim)
    ids = torch.tensor([[10, 0, 3]], device=dev)
    out = torch.empty(1, 3, dim, device=dev)
    gx, gh = layer_ops.residual_norm(None, None, w.to(dev, F32), 1e-4, dtype, embed=table.to(dev, dtype), ids=ids, embed_scale=3.3, x_out=out)
    assert gx is out and hm.rms_error(out.cpu()[0], 3.3 * table[[10, 0, 3]]) < 1e-6
    assert hm.rms_error(gh.cpu()[0], ho.rms_norm(3.3 * table[[10, 0, 3]], 1e-4, w)) < (1e-6 if dtype == F32 else 3e-3)


@pytest.mark.parametrize("rows,K,N,n", [(1, 40, 24, 1), (1, 2056, 99, 5), (4, 264, 17, 2), (2, 4096, 130, 70), (3, 72, 40, 64), (6, 64, 40, 3)])
@pytest.mark.parametrize("bias", [False, True])
def test_output_product_with_residual_sum_and_average(dev, rows, K, N, n, bias):
    from socket_amd import layer_ops
    g = torch.Generator().manual_seed(K + N)
    h, x, w = _rand(g, rows, 1, K), _rand(g, rows, 1, N), (_rand(g, N, K) / K ** 0.5).to(BF16).double()
    b = _rand(g, N) if bias else None
    past, dwa = _rand(g, n + 1, rows, 1, N), _rand(g, n + 1)
    res = x + h @ w.t() + (b if bias else 0)
    p = past.to(dev, F32)
    depth = layer_ops.Depth(p, n, dwa.to(dev, F32))
    bd = None if b is None else b.to(dev, BF16)
    y, pend = layer_ops.linear_residual(h.to(dev, BF16), w.to(dev, BF16), x.to(dev, F32), bd, depth)
    assert (pend is None) == (rows <= 4)
    if pend is not None:
        y, _ = layer_ops.residual_norm(y, pend, torch.ones(N, device=dev), 1e-4, BF16)
    tol = 1e-5 if rows <= 4 else 6e-3
    assert hm.rms_error(y.cpu(), go.depth_average(list(past[:n]) + [res], dwa)) < tol
    assert hm.rms_error(p[n].cpu(), res) < tol and torch.equal(p[:n].cpu().double(), past[:n])
    # without averaging: the plain residual sum
    if rows <= 4:
        y, _ = layer_ops.linear_residual(h.to(dev, BF16), w.to(dev, BF16), x.to(dev, F32), bd)
        assert hm.rms_error(y.cpu(), res) < tol


@pytest.mark.parametrize("rows,K,N", [(1, 40, 24), (1, 2056, 99), (3, 264, 17), (6, 64, 40)])
def test_decode_products_with_silu_unit_and_biases(dev, rows, K, N):
    from socket_amd import layer_ops
    g = torch.Generator().manual_seed(K + N)
    x, w = _rand(g, rows, 1, K), 1 + 0.2 * _rand(g, K)
    w1, w2 = ((_rand(g, N, K) / K ** 0.5).to(BF16).double() for _ in range(2))
    b1, b2 = _rand(g, N), _rand(g, N)
    h = ho.rms_norm(x, 1e-5, w)
    d = lambda t: t.to(dev, BF16)
    _, y = layer_ops.norm_linear(x.to(dev, F32), None, w.to(dev, F32), 1e-5, d(w1), up_weight=d(w2), act="silu", bias=d(b1), up_bias=d(b2))
    assert hm.rms_error(y.cpu(), ho.silu(h @ w1.t() + b1) * (h @ w2.t() + b2)) < 1.2e-2
    _, y = layer_ops.norm_linear(x.to(dev, F32), None, w.to(dev, F32), 1e-5, d(w1), bias=d(b1))
    assert hm.rms_error(y.cpu(), h @ w1.t() + b1) < 8e-3
    # a row that is a slice of a wider one
    wide = torch.zeros(rows, 1, K + 24, device=dev)
    wide[..., 8:8 + K] = x.to(dev, F32)
    wide[..., 8 + K:] = 1e6
    _, y = layer_ops.norm_linear(wide[..., 8:8 + K], None, w.to(dev, F32), 1e-5, d(w1), f32_out=True)
    assert hm.rms_error(y.cpu(), h @ w1.t()) < 8e-3


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("ff", [24, 21])
def test_silu_unit_and_tanh_rows(dev, dtype, ff):
    from socket_amd import layer_ops
    g = torch.Generator().manual_seed(ff)
    gu = 4 * _rand(g, 1, 5, 2 * ff)
    got = layer_ops.gated_unit(gu.to(dev, dtype), "silu").cpu()
    assert hm.rms_error(got, ho.silu(gu[..., :ff]) * gu[..., ff:]) < (1e-6 if dtype == F32 else 6e-3)
    x = gu.to(dtype).to(dev)
    x[0, 0, 0], x[0, 1, 0], x[0, 2, 0] = 1e-4, -90.0, 0.0499
    got = layer_ops.tanh_rows(x[..., :ff]).cpu().double()
    want = torch.tanh(x[..., :ff].cpu().double())
    assert ((got - want).abs() <= (3e-7 if dtype == F32 else 4e-3) * want.abs().clamp(min=0.05)).all() or \
        float((got - want).abs().max()) < (3e-7 if dtype == F32 else 4e-3)


# ---- generalized delta rule ----------------------------------------------------------------------------

def _branch(dev, dtype, heads, dim, rank, seed, decay_shift=0.0, rate_shift=0.0):
    from socket_amd import guselix
    from socket_amd.mixers import ColumnMap, GatedRecurrence
    g = torch.Generator().manual_seed(seed)
    cols = ColumnMap()
    br = GatedRecurrence(guselix.general_delta(heads, dim, rank), 32, 1e-4, cols, "r")
    vals = {}
    for n, p in br.named_parameters():
        t = _rand(g, *p.shape)
        t = {"decay_w": lambda: t / rank ** 0.5, "decay_bias": lambda: 2 * t - 2 + decay_shift, "rate_bias": lambda: t + rate_shift,
             "norm": lambda: 1 + 0.2 * t}.get(n, lambda: t)()
        vals[n] = t.to(BF16).double()
        p.data = vals[n].to(dev, F32 if n in br.FP32 else dtype)
    return br, cols, vals


def _branch_oracle(br, cols, vals, proj):
    c, T = br.spec, proj.shape[0]
    col = {n.split(".")[1]: proj[:, o:o + cols.rows[n]] for n, o in cols.offset.items()}
    r, k, v = (col[n].reshape(T, c.heads, c.dim) for n in "qkv")
    z = torch.tanh(col["a1"]) @ vals["decay_w"].t() + vals["decay_bias"]
    a = ho.sigmoid(col["rate"] + vals["rate_bias"])
    o, S = go.general_delta_rule(r, k, v, go.decay_factor(z).view_as(r), a.view_as(r))
    o = ho.rms_norm(o, 1e-4).reshape(T, -1) * vals["norm"] * ho.sigmoid(col["g"])
    return o, S


GENERAL = [  # heads, dim, decay rank, decay shift, rate shift
    (4, 16, 12, 0.0, 0.0),
    (2, 64, 16, 0.0, 0.0),
    (3, 48, 64, 30.0, 0.0),      # every channel at the strongest decay: 64 tokens span 2^56
    (2, 32, 136, -30.0, 30.0),   # no decay at all, full removal
    (3, 9, 7, 0.0, 0.0),         # scalar paths
    (1, 1, 1, 1.0, 0.0),
    (5, 40, 8, 1.0, -30.0),      # no removal
    (1, 80, 24, 0.0, 0.0),       # 32-token chunks
    (1, 128, 128, 30.0, 1.0),
    (1, 200, 16, 0.0, 0.0),      # values staged late
    (1, 256, 16, 0.0, 0.0),
]


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("case", range(len(GENERAL)))
def test_general_delta_in_portions_and_steps(dev, dtype, case):
    from socket_amd.mixers import StepContext
    heads, dim, rank, ds, rs = GENERAL[case]
    br, cols, vals = _branch(dev, dtype, heads, dim, rank, case, ds, rs)
    B, cuts, tail = 2, (70, 2, 3, 129), 5
    T = sum(cuts) + tail
    g = torch.Generator().manual_seed(11)
    proj = _rand(g, B, T, cols.total)
    k_at = cols.offset["r.k"]
    n = heads * dim
    proj[..., k_at:k_at + n] = (proj[..., k_at:k_at + n] * 1.3 / dim ** 0.5).to(BF16).double()
    proj[:, T - 3, k_at:k_at + n] = proj[:, 5, k_at:k_at + n]       # a key that comes back far away
    want = [_branch_oracle(br, cols, vals, proj[b]) for b in range(B)]
    p = proj.to(dev, dtype)
    br.alloc_state(B, T, dtype, dev)
    br.state.s.fill_(7.0)          # left over from someone else: a portion at position 0 starts anew
    outs = []
    for plan in ((T,), cuts + (1,) * tail, (2,) * (T // 2) + (1,) * (T % 2)):
        out, at = [], 0
        for m in plan:
            pos = torch.tensor([at], device=dev) if (m == 1 and at > 0) else None
            out.append(br.heads(p[:, at:at + m], StepContext(None if pos is not None else at, pos, {})))
            at += m
        outs.append(torch.cat(out, 1).cpu())
        S = br.state.s.cpu()
        for b in range(B):
            assert hm.rms_error(S[b].flatten(1), want[b][1].flatten(1)) < (3e-5 if dtype == F32 else 2e-2), (plan, b)
    w = torch.stack([x[0] for x in want])
    for got in outs:
        assert torch.isfinite(got.float()).all()
        assert hm.rms_error(got, w) < (1e-4 if dtype == F32 else 5e-2)
        assert hm.mean_error(got, w) < (1e-5 if dtype == F32 else 1e-2)


def test_general_delta_long_decoding_and_segments(dev, monkeypatch):
    from socket_amd import layer_ops
    from socket_amd.mixers import StepContext
    br, cols, vals = _branch(dev, F32, 2, 24, 12, 5)
    T = 400
    proj = _rand(torch.Generator().manual_seed(1), 1, T, cols.total)
    want, S = _branch_oracle(br, cols, vals, proj[0])
    p = proj.to(dev, F32)
    br.alloc_state(1, T, F32, dev)
    one = br.heads(p, StepContext(0, None, {}))
    assert hm.rms_error(one[0].cpu(), want) < 1e-4
    monkeypatch.setattr(layer_ops, "SCAN_SEGMENT", 128)
    assert hm.rms_error(br.heads(p, StepContext(0, None, {}))[0].cpu(), want) < 1e-4
    out = [br.heads(p[:, :2], StepContext(0, None, {}))]
    for t in range(2, T):
        out.append(br.heads(p[:, t:t + 1], StepContext(None, torch.tensor([t], device=dev), {})))
    assert hm.rms_error(torch.cat(out, 1)[0].cpu(), want) < 1e-4
    assert hm.rms_error(br.state.s[0].cpu().flatten(1), S.flatten(1)) < 2e-5


def test_general_delta_refuses_decays_it_cannot_split(dev):
    from socket_amd import _lib
    from socket_amd.mixers import StepContext
    br, cols, _ = _branch(dev, F32, 1, 16, 8, 0)
    br.spec.decay_rate = 1.2       # 64 tokens: past 2^100
    br.alloc_state(1, 4, F32, dev)
    with pytest.raises(_lib.SocketHipError):
        br.heads(torch.zeros(1, 4, cols.total, device=dev), StepContext(0, None, {}))


# ---- latent attention ----------------------------------------------------------------------------------

LATENT = [  # heads, dim, rot, vdim, q_rank, kv_rank, scale
    (3, 16, 8, 24, 40, 32, 0.3),
    (5, 9, 6, 19, 13, 11, 0.4),            # scalar paths, padded cache rows
    (1, 1, 2, 1, 1, 1, 1.0),
    (2, 72, 24, 96, 48, 96, 0.15),         # values wider than the unrotated keys
    (17, 48, 16, 40, 64, 104, 0.2),        # more heads than a tile
    (2, 96, 32, 128, 64, 160, 0.12),
    (2, 128, 64, 128, 96, 256, 0.1),
    (16, 128, 64, 96, 72, 512, 0.08),
    (2, 120, 128, 200, 40, 384, 0.07),
    (1, 300, 20, 280, 40, 600, 0.05),      # past the matrix-core forms
]


def _latent_branch(dev, dtype, case, width=32):
    from socket_amd.mixers import ColumnMap, LatentAttention, LatentAttentionSpec
    H, dim, rot, vdim, qr, kr, scale = LATENT[case]
    g = torch.Generator().manual_seed(case)
    cols = ColumnMap()
    br = LatentAttention(LatentAttentionSpec(H, dim, rot, vdim, qr, kr, 500.0, scale), width, 1e-4, cols, "a")
    vals = {}
    for n, p in br.named_parameters():
        t = _rand(g, *p.shape)
        t = 1 + 0.2 * t if n.endswith("norm") else t * (1.5 if n == "uq" else 1.0) / p.shape[1] ** 0.5
        vals[n] = t.to(BF16).double()
        p.data = vals[n].to(dev, F32 if n in br.FP32 else dtype)
    return br, cols, vals


def _latent_oracle(br, cols, vals, proj, gate=True):
    c, T = br.spec, proj.shape[0]
    col = {n.split(".")[1]: proj[:, o:o + cols.rows[n]] for n, o in cols.offset.items()}
    q = (ho.rms_norm(col["cq"], 1e-4, vals["q_norm"]) @ vals["uq"].t()).view(T, c.heads, -1)
    lat = ho.rms_norm(col["c"], 1e-4, vals["c_norm"])
    n = c.heads * c.dim
    o = go.latent_attention(q, lat, col["rot"], vals["ukv"][:n], vals["ukv"][n:], c.heads, c.dim, c.scale, c.rot_base)
    return o.reshape(T, -1) * ho.sigmoid(col["g"])


def _far_keys(br, cols, vals, proj, pairs):
    """Rewrite rows so that the query at `t` finds the key at `j`: the latent of j and the shared part
    point along what head 0's query of t asks for (in the frame of the two positions)."""
    c = br.spec
    for t, j in pairs:
        q = (ho.rms_norm(proj[t, cols.offset["a.cq"]:cols.offset["a.cq"] + c.q_rank], 1e-4, vals["q_norm"]) @ vals["uq"].t()).view(c.heads, -1)[0]
        want = q[:c.dim] @ vals["ukv"][:c.dim]
        at = cols.offset["a.c"]
        proj[j, at:at + c.kv_rank] = (3 * want / want.norm() * c.kv_rank ** 0.5).to(BF16).double()
        # turn the shared part by t - j, so that after both rotations it meets the query's
        r = ho.rotary(q[None, None, c.dim:], torch.tensor([t - j]), c.rot_dim, c.rot_base)[0, 0]
        at = cols.offset["a.rot"]
        proj[j, at:at + c.rot_dim] = (4 * r / max(float(r.norm()), 1e-3)).to(BF16).double()


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("case", range(len(LATENT)))
def test_latent_attention_in_portions_and_steps(dev, dtype, case):
    from socket_amd.mixers import StepContext
    from socket_amd.model import precompute_freqs_cis
    br, cols, vals = _latent_branch(dev, dtype, case)
    c = br.spec
    B, T = 2, 210
    g = torch.Generator().manual_seed(case)
    proj = _rand(g, B, T, cols.total)
    for b in range(B):
        _far_keys(br, cols, vals, proj[b], [(T - 1, 1), (T - 2, 16), (T - 4, 63), (T - 5, 64), (150, 0), (80, 79)])
    want = torch.stack([_latent_oracle(br, cols, vals, proj[b]) for b in range(B)])
    ctx_rope = {br.rope_key(): precompute_freqs_cis(T + 300, c.rot_dim, c.rot_base, dtype=F32).to(dev)}
    br.alloc_state(B, T + 300, dtype, dev)
    br.state.rows.fill_(float("nan"))       # what was never written must never count
    p = proj.to(dev, dtype)
    for plan in ((T,), (100, 2, 8, 9, 7, 70, 2) + (1,) * 12, (3, 1, 1, 1) + (2,) * 102):
        out, at = [], 0
        for m in plan:
            pos = torch.tensor([at], device=dev) if (m == 1 and at > 0) else None
            x = p[:, at:at + m]
            if pos is not None:
                x = x.float()               # a decode step's projected row is fp32
            out.append(br.heads(x, StepContext(None if pos is not None else at, pos, ctx_rope)))
            at += m
        assert at == T
        got = torch.cat(out, 1).cpu()
        assert torch.isfinite(got.float()).all()
        assert hm.rms_error(got, want) < (1e-5 if dtype == F32 else 4e-2), plan
        assert hm.mean_error(got, want) < (3e-6 if dtype == F32 else 1e-2), plan


def test_far_key_decides_a_long_decode_step(dev):
    """Thousands of cache rows dealt to many workgroups, one of them asked for; the recorded far key
    outweighs the rest, wherever in a tile or split it lies."""
    from socket_amd import layer_ops
    from socket_amd.sequence_state import LatentCache
    H, rank, rot, vdim, T = 16, 512, 64, 64, 5000
    g = torch.Generator().manual_seed(3)
    cache = LatentCache(1, 6000, rank, rot, BF16, dev)
    rows = _rand(g, T, rank + rot)
    cache.rows[0, :T] = rows.to(dev, BF16)
    cache.rows[0, T:] = float("nan")
    uv = (_rand(g, H * vdim, rank) / rank ** 0.5).to(BF16)
    for j in (0, 15, 16, 2047, 2048, 4095, T - 1):
        q = _rand(g, H, rank + rot)
        q[5] = (rows[j] * 0.9).to(BF16).double()
        s = (q @ rows.t()) * 0.02
        pr = torch.softmax(s, -1)
        assert pr[5, j] > 0.5
        want = torch.stack([uv.double()[h * vdim:(h + 1) * vdim] @ (pr[h] @ rows[:, :rank]) for h in range(H)]).reshape(1, -1)
        for kw in (dict(pos=torch.tensor([T - 1], device=dev)), dict(pos0=T - 1), dict(pos0=T - 1, force_simple=True)):
            got = layer_ops.latent_attend(q.to(dev, BF16)[None, None], cache, 0.02, uv.to(dev), vdim, None, **kw)
            assert hm.rms_error(got[0].cpu(), want) < (8e-3 if "force_simple" not in kw else 1.5e-2), (j, kw)


@pytest.mark.parametrize("H,D,D2,dv", [(2, 40, 24, 64), (3, 64, 32, 88), (2, 96, 32, 72), (4, 128, 64, 128), (1, 184, 72, 256), (2, 64, 8, 128)])
def test_causal_attention_kernels_agree(dev, H, D, D2, dv):
    """Shared second key segment, values of another width, positions before the portion, the gate."""
    from socket_amd import layer_ops
    g = torch.Generator().manual_seed(D)
    B, S, T = 2, 330, 201
    q, k, ks, v = _rand(g, B, T, H, D + D2), _rand(g, B, S, H, D), _rand(g, B, S, D2), _rand(g, B, S, H, dv)
    gate = _rand(g, B, T, H * dv)
    q[:, -1, 0] = 2 * torch.cat([k[:, 2, 0], ks[:, 2]], -1)         # a far key, and one at a tile's edge
    q[:, -2, 0] = 2 * torch.cat([k[:, 64, 0], ks[:, 64]], -1)
    scale = (D + D2) ** -0.5
    d = [t.to(dev, BF16) for t in (q, k, ks, v)]
    mma = layer_ops.causal_attend(*d, S - T, scale, gate.to(dev, BF16))
    simple = layer_ops.causal_attend(*d, S - T, scale, gate.to(dev, BF16), force_simple=True)
    exact = layer_ops.causal_attend(*[t.to(dev, F32) for t in (q, k, ks, v)], S - T, scale, gate.to(dev, F32))
    full = torch.cat([torch.zeros(B, S - T, H, D + D2, dtype=torch.float64), q], 1)
    want = torch.stack([go.causal_softmax_attention(full[b], torch.cat([k[b], ks[b][:, None].expand(S, H, D2)], -1), v[b], scale)[S - T:]
                        for b in range(B)]) * ho.sigmoid(gate).view(B, T, H, dv)
    for got, tol in ((mma, 8e-3), (simple, 8e-3), (exact, 3e-6)):
        assert _row_error(got.cpu().flatten(2), want.flatten(2)) < tol


# ---- whole models -----------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("name", list(gm.CONFIGS))
def test_model_whole_portions_and_token_by_token(dev, tmp_path, dtype, name):
    cfg = gm.CONFIGS[name]
    w = gm.weights(cfg, seed=len(name))
    m = hm.build(tmp_path, cfg, w, dev, dtype)
    T = 90
    m.setup_caches(1, T)
    tok = hm.tokens(T, cfg["vocab"], 1)
    collect = []
    want = go.forward(w, cfg, tok, collect)
    rng = random.Random(4)
    cuts = []
    while sum(cuts) < T:
        cuts.append(min(rng.choice([2, 3, 7, 24, 1]), T - sum(cuts)))
    for plan in ((T,), (1,) * T, tuple(cuts), (2,) * (T // 2), (T - 20,) + (1,) * 20):
        got = _feed(m, tok, plan, dev)
        assert hm.rms_error(got, want) < TOL[dtype], plan
        assert hm.mean_error(got, want) < MEAN_TOL[dtype], plan
    for step in (False, True):
        got = []
        if step:
            _feed(m, tok[:T - 1], (T - 1,), dev)
            m._run(torch.tensor([tok[T - 1:]], device=dev), torch.tensor([T - 1], device=dev), False, None, False, None, got)
        else:
            m._run(torch.tensor([tok], device=dev), torch.arange(T, device=dev), False, 0, False, None, got)
        assert len(got) == len(collect)
        for a, b in zip(got, collect):
            assert hm.rms_error(a[0].cpu(), b[T - 1:] if step else b) < TOL[dtype]


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_model_batch_equals_each_alone_and_state_is_reused(dev, tmp_path, dtype):
    cfg = gm.CONFIGS["mixed"]
    w = gm.weights(cfg, seed=9, decay_shift=1.0)
    m = hm.build(tmp_path, cfg, w, dev, dtype)
    T = 60
    toks = [hm.tokens(T, cfg["vocab"], s) for s in (1, 2, 3, 4, 5)]
    want = torch.stack([go.forward(w, cfg, t) for t in toks])
    for B in (3, 5):                         # (five rows: past the matrix-vector kernel)
        for cuts in ((T,), (31, 2, 3) + (1,) * 24):
            m.setup_caches(B, T)
            assert hm.rms_error(_feed(m, toks[:B], cuts, dev), want[:B]) < TOL[dtype]
    # one request after another in the same slots: a long one, a one-token one, short ones
    m.setup_caches(1, 200)
    for seed, n in ((6, 150), (7, 1), (8, 30), (6, 3)):
        tok = hm.tokens(n, cfg["vocab"], seed)
        cuts = (n - 2, 1, 1) if n > 3 else (n,)
        assert hm.rms_error(_feed(m, tok, cuts, dev), go.forward(w, cfg, tok)) < TOL[dtype], n


def test_model_of_many_layers_averages_over_all_of_them(dev, tmp_path):
    """More results than a wave has lanes."""
    cfg = gm.config([gm.delta_layer(gm.delta(1, 8)) for _ in range(70)], width=16, vocab=31)
    w = gm.weights(cfg, seed=2, decay_rank=3)
    for i in range(70):
        w[f"l{i}.dwa"] = (0.5 * w[f"l{i}.dwa"] / (i + 2) ** 0.5).to(BF16).double()
        w[f"l{i}.dwa"][-1] = 0.75
        w[f"l{i}.dwa"][0] = 0.25
    tok = hm.tokens(12, 31, 3)
    want = go.forward(w, cfg, tok)
    for dtype in (F32, BF16):
        m = hm.build(tmp_path / str(dtype), cfg, w, dev, dtype)
        m.setup_caches(1, 12)
        for cuts in ((12,), (4,) + (1,) * 8):
            got = _feed(m, tok, cuts, dev)
            assert hm.rms_error(got, want) < 3 * TOL[dtype], (dtype, cuts)


def test_model_refuses_what_would_corrupt_its_state(dev, tmp_path):
    cfg = gm.CONFIGS["mixed"]
    m = hm.build(tmp_path, cfg, gm.weights(cfg), dev, F32)
    m.setup_caches(1, 20)
    t = torch.tensor([[1, 2, 3]], device=dev)
    m(t, torch.arange(3, device=dev), pos0=0)
    with pytest.raises(RuntimeError, match="does not continue"):
        m(t, torch.arange(7, 10, device=dev), pos0=7)
    with pytest.raises(RuntimeError, match="out of bounds"):
        m(t, torch.arange(18, 21, device=dev), pos0=18)
    with pytest.raises(ValueError, match="sparse"):
        m.sparse_forward(t, torch.arange(3, device=dev), pos0=0)


def _greedy(w, cfg, tok, n):
    tok, margin = list(tok), []
    for _ in range(n):
        lg = go.forward(w, cfg, tok)[-1]
        top = torch.topk(lg, 2).values
        margin.append(float(top[0] - top[1]))
        tok.append(int(lg.argmax()))
    return tok, min(margin)


@pytest.mark.parametrize("graph,portion", [(True, 0), (False, 0), (True, 7)])
def test_greedy_generation(dev, tmp_path, graph, portion):
    """generate() with and without a recorded decode step against the oracle's greedy continuation; the
    recorded step equals the eager one and leaves the state alone."""
    from socket_amd import generate as gen
    cfg = gm.CONFIGS["mixed"]
    w = gm.weights(cfg, seed=21)
    m = gen.load_model(hm.save(tmp_path, cfg, w), dev, F32)
    prompt, n = hm.tokens(19, cfg["vocab"], 5), 40
    want, margin = _greedy(w, cfg, prompt, n)
    assert margin > 1e-3, "pick another seed: a near tie decides nothing"
    seq, st = gen.generate(m, torch.tensor([prompt, prompt], device=dev), n, decode_type="dense", use_graph=graph,
                           check_graph=graph, prefill_portion=portion)
    assert seq.tolist() == [want, want]
    if graph:
        assert st["graph_check"]["same_token"] and st["graph_check"]["max_abs_logit_diff"] < 1e-4


def test_recorded_step_in_16_bit_equals_the_eager_one(dev, tmp_path):
    from socket_amd import generate as gen
    cfg = gm.CONFIGS["wide"]
    m = gen.load_model(hm.save(tmp_path, cfg, gm.weights(cfg, seed=6)), dev, BF16)
    prompt = torch.tensor([hm.tokens(50, cfg["vocab"], 5)], device=dev)
    _, st = gen.generate(m, prompt, 12, decode_type="dense", use_graph=True, check_graph=True)
    assert st["graph_check"]["same_token"] and st["graph_check"]["max_abs_logit_diff"] == 0.0


def test_command_line_generates_from_a_model_folder(dev, tmp_path):
    cfg = gm.CONFIGS["odd"]
    w = gm.weights(cfg, seed=2)
    path = hm.save(tmp_path, cfg, w)
    prompt = hm.tokens(9, cfg["vocab"], 5)
    want, margin = _greedy(w, cfg, prompt, 12)
    assert margin > 1e-3
    r = subprocess.run([sys.executable, "-m", "socket_amd.generate", "--model", path, "--dtype", "float32", "--prompt_tokens",
                        ",".join(map(str, prompt)), "--max_new_tokens", "12", "--print_tokens"], cwd=ROOT, capture_output=True,
                       text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert json.loads(r.stdout.splitlines()[-1])["dense"]["tokens"] == [want[9:]]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_run(dev, tmp_path, dtype):
    cfg = gm.CONFIGS["wide"]
    w = gm.weights(cfg, seed=4)
    path = hm.save(tmp_path / "m", cfg, w)
    out = tmp_path / "out"
    out.mkdir()
    steps, want = [], {}
    for name, n, cuts in (("a", 80, (60, 2, 1, 1, 16)), ("b", 1, (1,)), ("c", 45, (41, 1, 1, 1, 1))):
        tok = hm.tokens(n, cfg["vocab"], n)
        ref = go.forward(w, cfg, tok)
        at = 0
        for k in cuts:
            places = [p for p in range(k) if (at + p) % 3 == 0 or k == 1]
            i = len(steps)
            steps.append({"step": i, "entries": [{"id": name, "tokens": tok[at:at + k], "want": places}],
                          "end": [name] if at + k == n else []})
            if places:
                want[i] = ref[[at + p for p in places]]
            at += k
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", dtype, "--out", str(out),
                        "--max-tokens", "80"], input="\n".join(map(json.dumps, steps)) + "\n", capture_output=True, text=True,
                       timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [ln for ln in r.stdout.splitlines() if ln.startswith("done")] == [f"done {i}" for i in range(len(steps))]
    for i in range(len(steps)):
        f = out / f"{i}.f32"
        assert f.exists() == (i in want)
        if i in want:
            got = torch.from_numpy(np.fromfile(f, dtype="<f4").reshape(want[i].shape))
            assert hm.rms_error(got, want[i]) < TOL[getattr(torch, dtype)], i
