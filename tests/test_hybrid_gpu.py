"""The hybrid decoders on the device against the plain restatement in
oracle/hybrid_oracle.py: each mechanism alone, then whole models in portions, token by
token, in batches, in reused state, and through generate() and bin/trace_run."""
import json
import os
import random
import subprocess
import sys

import numpy as np
import pytest
import torch

from oracle import hybrid_oracle as ho
from tests import hybrid_models as hm

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
TOL = {torch.float32: 2e-5, torch.bfloat16: 8e-2}     # of the worst token
MEAN_TOL = {torch.float32: 1e-5, torch.bfloat16: 3e-2}


def _rand(g, *shape, dtype=torch.float64):
    return torch.randn(*shape, generator=g, dtype=torch.float64).to(torch.bfloat16).to(dtype)


# ---- rows ------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("rows,dim,two,post", [(1, 40, True, True), (5, 37, False, True), (3, 2056, True, False), (2, 8192, True, True)])
def test_residual_norm(dev, dtype, rows, dim, two, post):
    from socket_amd import layer_ops
    g = torch.Generator().manual_seed(dim)
    x, a, b = _rand(g, rows, dim), _rand(g, rows, dim), _rand(g, rows, dim)
    pw, w = 1 + 0.2 * _rand(g, dim), 1 + 0.2 * _rand(g, dim)
    y = 0.7 * a + (1.3 * b if two else 0)
    want_x = x + (ho.rms_norm(y, 1e-4, pw) if post else y)
    want_h = ho.rms_norm(want_x, 1e-4, w)
    pend = layer_ops.Pending(a.to(dev, dtype), 0.7, b.to(dev, dtype) if two else None, 1.3 if two else 0.0,
                             pw.to(dev, torch.float32) if post else None)
    gx, gh = layer_ops.residual_norm(x.to(dev, torch.float32), pend, w.to(dev, torch.float32), 1e-4, dtype)
    assert gx.dtype == torch.float32 and hm.rms_error(gx.cpu(), want_x) < 1e-6
    assert gh.dtype == dtype and hm.rms_error(gh.cpu(), want_h) < (1e-6 if dtype == torch.float32 else 3e-3)
    # the stream starts at rows of the embedding (int32 and int64 ids)
    table = _rand(g, 11, dim)
    for idt in (torch.int32, torch.int64):
        ids = torch.tensor([[10, 0, 3]], dtype=idt, device=dev)
        gx, gh = layer_ops.residual_norm(None, None, w.to(dev, torch.float32), 1e-4, dtype, embed=table.to(dev, dtype), ids=ids)
        assert torch.equal(gx.cpu().double()[0], table[[10, 0, 3]])
        assert hm.rms_error(gh.cpu()[0], ho.rms_norm(table[[10, 0, 3]], 1e-4, w)) < (1e-6 if dtype == torch.float32 else 3e-3)


@pytest.mark.parametrize("rows,K,N", [(1, 40, 24), (1, 2056, 99), (4, 264, 17), (2, 4096, 130), (6, 64, 40)])
def test_decode_products_with_norm_gate_and_two_terms(dev, rows, K, N):
    from socket_amd import layer_ops
    bf = torch.bfloat16
    g = torch.Generator().manual_seed(K + N)
    x, a = _rand(g, rows, 1, K), _rand(g, rows, 1, K)
    w1, w2, wk = _rand(g, N, K) / K ** 0.5, _rand(g, N, K) / K ** 0.5, _rand(g, N, 2 * K) / K ** 0.5
    w1, w2, wk = (t.to(bf).double() for t in (w1, w2, wk))
    pw, w = 1 + 0.2 * _rand(g, K), 1 + 0.2 * _rand(g, K)
    f32 = dict(device=dev, dtype=torch.float32)
    pend = layer_ops.Pending(a.to(**f32), 1.0, post_w=pw.to(**f32))
    want_x = x + ho.rms_norm(a, 1e-5, pw)
    h = ho.rms_norm(want_x, 1e-5, w)
    gx, y = layer_ops.norm_linear(x.to(**f32), pend, w.to(**f32), 1e-5, w1.to(dev, bf), f32_out=True)
    assert y.dtype == torch.float32 and hm.rms_error(gx.cpu(), want_x) < 1e-6 and hm.rms_error(y.cpu(), h @ w1.t()) < 6e-3
    lim = 0.8
    u = torch.clamp(h @ w2.t(), -lim, lim)
    t = torch.clamp(h @ w1.t(), max=lim)
    _, y = layer_ops.norm_linear(x.to(**f32), pend, w.to(**f32), 1e-5, w1.to(dev, bf), up_weight=w2.to(dev, bf), limit=lim)
    assert hm.rms_error(y.cpu(), t * ho.sigmoid(1.702 * t) * (u + 1)) < 1.2e-2
    b = _rand(g, rows, 1, 2 * K)
    p = layer_ops.linear_terms([(a.to(dev, bf), w1.to(dev, bf), 0.8), (b.to(dev, bf), wk.to(dev, bf), -1.5)])
    got = p.scale_a * p.a.double() + (p.scale_b * p.b.double() if p.b is not None else 0)
    assert hm.rms_error(got.cpu(), 0.8 * a @ w1.t() - 1.5 * b @ wk.t()) < 6e-3
    one = layer_ops.linear_f32(a.to(dev, bf), w1.to(dev, bf))
    assert one.dtype == torch.float32 and hm.rms_error(one.cpu(), a @ w1.t()) < 1e-5


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("ff", [24, 21])
def test_clamped_glu_beyond_its_limits(dev, dtype, ff):
    from socket_amd import layer_ops
    g = torch.Generator().manual_seed(ff)
    gu = 4 * _rand(g, 3, 2 * ff)
    t, u = torch.clamp(gu[:, :ff], max=1.5), torch.clamp(gu[:, ff:], -1.5, 1.5)
    assert (gu[:, :ff] > 1.5).any() and (gu[:, :ff] < -4).any() and (gu[:, ff:] < -1.5).any()
    got = layer_ops.gated_unit(gu.to(dev, dtype), "clamped", 1.5).cpu()
    assert hm.rms_error(got, t * ho.sigmoid(1.702 * t) * (u + 1)) < (1e-6 if dtype == torch.float32 else 4e-3)


# ---- rotary and chunked attention ------------------------------------------------------------------

def _ring(dev, dtype, B, G, D, chunk, cap=4096):
    from socket_amd.sequence_state import ChunkRing
    r = ChunkRing(B, cap, G, D, chunk, dtype, dev)
    r.k.fill_(float("nan"))     # what was never written must never count
    r.v.fill_(float("nan"))
    return r


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("D,rot", [(16, 16), (24, 8), (10, 6), (64, 32), (8, 0)])
def test_rotate_half_rows_and_ring_append(dev, dtype, D, rot):
    from socket_amd import layer_ops
    from socket_amd.model import precompute_freqs_cis
    B, T, H, G, chunk, pos0 = 2, 7, 4, 2, 5, 901
    g = torch.Generator().manual_seed(D)
    proj = _rand(g, B, T, 8 + (H + G) * D + 8)
    table = precompute_freqs_cis(1000, rot, 300.0, dtype=torch.float32).to(dev)
    q_off, k_off = 8, 8 + H * D
    want_q = torch.stack([ho.rotary(proj[b, :, q_off:k_off].view(T, H, D), pos0 + torch.arange(T), rot, 300.0) for b in range(B)])
    want_k = torch.stack([ho.rotary(proj[b, :, k_off:k_off + G * D].view(T, G, D), pos0 + torch.arange(T), rot, 300.0)
                          for b in range(B)])
    p = proj.to(dev, dtype)
    q, k = layer_ops.rope_half(p, q_off, k_off, H, G, D, rot, table, pos0=pos0)
    tol = 2e-6 if dtype == torch.float32 else 4e-3
    assert hm.rms_error(q.cpu(), want_q) < tol and hm.rms_error(k.cpu(), want_k) < tol
    ring = _ring(dev, dtype, B, G, D, chunk)
    for t in (0, 3, 6):
        pos = torch.tensor([pos0 + t], device=dev)
        q1 = layer_ops.rope_half(p[:, t:t + 1], q_off, k_off, H, G, D, rot, table, pos=pos, ring=ring, q_pitch=D + 8)
        slot = (pos0 + t) % chunk
        assert torch.equal(q1[..., :D], q[:, t:t + 1]) and (q1[..., D:] == 0).all()
        assert torch.equal(ring.k[:, :, slot], k[:, t]) and torch.equal(ring.v[:, :, slot].reshape(B, -1), p[:, t, k_off:k_off + G * D])
        assert ring.len.tolist() == [slot + 1] * B


def _attend_case(dev, dtype, H, G, D, chunk, cuts, softcap, scale, seed, simple=False, B=2, decode_tail=0):
    """Portions `cuts`, then decode steps, through one ring; returns (got, want) [B,T,H,D]."""
    from socket_amd import layer_ops
    g = torch.Generator().manual_seed(seed)
    T = sum(cuts) + decode_tail
    q, k, v = _rand(g, B, T, H, D), _rand(g, B, T, G, D), _rand(g, B, T, G, D)
    # keys that stand out for queries just inside and just outside a chunk's edge, for the last
    # position and for one far inside the chunk
    for e in range(chunk, T, chunk):
        k[:, e - 1] = 2.5 * q[:, min(e, T - 1), ::H // G]         # outside: the next chunk's first query must not see it
        k[:, e] = 2.5 * q[:, min(e + chunk - 1, T - 1), ::H // G]  # inside: the last query of the chunk must see its first key
    if T > 8:
        k[:, T // 2] = 2.5 * q[:, T - 1, ::H // G]
    k = k.to(torch.bfloat16).double()
    want = torch.stack([ho.chunked_attention(q[b], k[b], v[b], scale, softcap if softcap else 1e9, chunk) for b in range(B)])
    ring = _ring(dev, dtype, B, G, D, chunk)
    qd, kd, vd = (t.to(dev, dtype) for t in (q, k, v))
    out, at = [], 0
    for n in cuts:
        sl = slice(at, at + n)
        out.append(layer_ops.chunk_attend(qd[:, sl], kd[:, sl], vd[:, sl], ring, at, scale, softcap, force_simple=simple))
        at += n
    for t in range(at, T):
        slot = t % chunk
        ring.k[:, :, slot], ring.v[:, :, slot] = kd[:, t], vd[:, t]
        ring.len.fill_(slot + 1)
        # (rows past the visible prefix belong to an older chunk or to nobody)
        out.append(layer_ops.chunk_attend_step(qd[:, t:t + 1].contiguous(), ring, torch.tensor([t], device=dev), G, scale, softcap))
    return torch.cat(out, 1).cpu(), want


ATT = [  # H, G, D, chunk, cuts, softcap, scale
    (4, 2, 16, 24, (50, 2, 3, 40), 15.0, 0.25),
    (5, 1, 10, 13, (30, 2, 2, 20), 4.0, 0.4),         # scalar kernel: D not a multiple of 8
    (6, 2, 40, 64, (64, 64, 2, 70), 0.0, 0.2),        # no cap; portions that end at a chunk's edge
    (3, 3, 64, 200, (130, 70, 137), 90.0, 0.125),     # a cap too high for the maximum-free form
    (8, 1, 96, 80, (81, 79, 30), 25.0, 0.11),
    (8, 2, 128, 150, (149, 2, 200), 30.0, 0.09),
    (2, 1, 160, 40, (70, 31), 10.0, 0.1),
    (2, 2, 248, 70, (90, 2, 9), 50.0, 0.06),
]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("case", range(len(ATT)))
def test_chunk_attention_in_portions_and_steps(dev, dtype, case):
    H, G, D, chunk, cuts, cap, scale = ATT[case]
    got, want = _attend_case(dev, dtype, H, G, D, chunk, cuts, cap, scale, case, decode_tail=chunk + 3 if chunk < 100 else 12)
    assert torch.isfinite(got.float()).all()
    assert hm.rms_error(got, want) < (3e-6 if dtype == torch.float32 else 8e-3)


def test_chunk_attention_kernels_agree_and_see_a_long_chunk(dev):
    """Several key tiles and several splits of a decode step; one far key outweighs hundreds."""
    from socket_amd import layer_ops
    H, G, D, chunk, T = 8, 2, 128, 1500, 1400
    g = torch.Generator().manual_seed(7)
    q, k, v = _rand(g, 1, T, H, D), _rand(g, 1, T, G, D), _rand(g, 1, T, G, D)
    k[:, 3] = 1.5 * q[:, T - 1, ::H // G]
    k[:, 700] = 1.5 * q[:, T - 2, ::H // G]
    d = [t.to(dev, torch.bfloat16) for t in (q, k, v)]
    ring = _ring(dev, torch.bfloat16, 1, G, D, chunk)
    mma = layer_ops.chunk_attend(*d, ring, 0, 0.09, 40.0)
    simple = layer_ops.chunk_attend(*d, ring, 0, 0.09, 40.0, force_simple=True)
    assert hm.rms_error(mma.cpu(), simple.cpu().double()) < 6e-3
    for t in (T - 1, T - 2):
        kk, vv = k[0, :t + 1].to(torch.bfloat16).double(), v[0, :t + 1]
        h = 0
        s = (kk[:, 0] @ q[0, t, h]) * 0.09
        p = torch.softmax(40.0 * torch.tanh(s / 40.0), 0)
        assert p[3 if t == T - 1 else 700] > 0.3
        assert hm.rms_error(mma[0, t, h].cpu()[None], (p @ vv[:, 0])[None]) < 8e-3
    ring.len.fill_(T)
    step = layer_ops.chunk_attend_step(d[0][:, T - 1:], ring, torch.tensor([T - 1], device=dev), G, 0.09, 40.0)
    assert hm.rms_error(step.cpu(), simple[:, T - 1:].cpu().double()) < 6e-3


# ---- recurrences -------------------------------------------------------------------------------------

def _recurrence(dev, dtype, spec, seed, decay_shift=0.0):
    """A GatedRecurrence branch with random weights and the oracle's view of it."""
    from socket_amd.mixers import ColumnMap, GatedRecurrence
    g = torch.Generator().manual_seed(seed)
    cols = ColumnMap()
    br = GatedRecurrence(spec, 32, 1e-4, cols, "r")
    vals = {}
    for n, p in br.named_parameters():
        t = _rand(g, *p.shape)
        if n in ("decay_w", "gate_w"):
            t = t / p.shape[1] ** 0.5
        if n == "decay_bias":
            t = t - 2.0 + decay_shift
        if n == "norm":
            t = 1 + 0.2 * t
        vals[n] = t.to(torch.bfloat16).double()
        p.data = vals[n].to(dev, torch.float32 if n in br.FP32 else dtype)
    return br, cols, vals


def _recurrence_oracle(spec, cols, vals, proj):
    c, T = spec, proj.shape[0]
    col = {n.split(".")[1]: proj[:, o:o + cols.rows[n]] for n, o in cols.offset.items()}
    q, k, v = col["q"], col["k"], col["v"]
    if c.taps:
        w = torch.split(vals["conv_w"].t(), [q.shape[1], k.shape[1], v.shape[1]])
        q, k, v = (ho.silu(ho.causal_conv(x, t)) for x, t in zip((q, k, v), w))
    q, k, v = q.reshape(T, c.kv_heads, c.dim), k.reshape(T, c.kv_heads, c.dim), v.reshape(T, c.heads, c.vdim)
    if c.unit_qk:
        q, k = ho.unit(q), ho.unit(k)
    q = (q * c.dim ** -0.5).repeat_interleave(c.heads // c.kv_heads, 1)
    k = k.repeat_interleave(c.heads // c.kv_heads, 1)
    z = (col["a1"] @ vals["decay_w"].t() + vals["decay_bias"]).view(T, c.heads, c.dim)
    if c.decay == "exp_softplus":
        dec = torch.exp(-torch.exp(vals["a_log"])[None, :, None] * ho.softplus(z))
    else:
        dec = ho.sigmoid(z) ** (1 / c.tau)
    o, S = ho.delta_rule(q, k, v, dec, ho.sigmoid(col["b"])) if c.delta else ho.gated_linear(q, k, v, dec)
    gate = col["g"] @ vals["gate_w"].t() if c.gate_rank else col["g"]
    gate = (ho.sigmoid if c.gate == "sigmoid" else ho.silu)(gate).view(T, c.heads, c.vdim)
    return (ho.rms_norm(o, 1e-4, vals["norm"]) * gate).reshape(T, -1), S


def _specs():
    from socket_amd.mixers import RecurrenceSpec as R
    return {
        "delta": (R(4, 2, 16, 24, 12, True, 4, True, gate_rank=20), 0.0),
        "delta_strong_decay": (R(2, 2, 32, 16, 8, True, 3, True, gate_rank=8), 6.0),    # e^{-pl} would overflow
        "delta_mixed_decay": (R(3, 1, 48, 32, 8, True, 2, True, gate_rank=8), 2.5),
        "delta_odd": (R(3, 3, 9, 5, 7, True, 1, True, gate_rank=3), 0.0),
        "delta_128": (R(2, 1, 128, 128, 16, True, 4, True, gate_rank=16), 0.0),
        "delta_96": (R(1, 1, 96, 64, 16, True, 4, True, gate_rank=16), 0.0),
        "delta_wide": (R(1, 1, 200, 40, 16, True, 5, True, gate_rank=16), 0.0),         # 32-token chunks
        "delta_256": (R(1, 1, 256, 256, 16, True, 3, True, gate_rank=16), 0.0),
        "gla": (R(3, 3, 16, 8, 12, False, decay="sigmoid_root", tau=8.0, gate="silu"), 0.0),
        "gla_fast_decay": (R(2, 2, 24, 40, 12, False, decay="sigmoid_root", tau=0.5, gate="silu"), -6.0),
        "gla_64": (R(2, 2, 64, 128, 12, False, decay="sigmoid_root", tau=16.0, gate="silu"), 0.0),
        "gla_wide": (R(1, 1, 144, 33, 9, False, decay="sigmoid_root", tau=2.0, gate="silu"), 0.0),
    }


NAMES = ["delta", "delta_strong_decay", "delta_mixed_decay", "delta_odd", "delta_128", "delta_96", "delta_wide", "delta_256",
         "gla", "gla_fast_decay", "gla_64", "gla_wide"]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("name", NAMES)
def test_recurrence_in_portions_and_steps(dev, dtype, name):
    from socket_amd.mixers import StepContext
    spec, shift = _specs()[name]
    br, cols, vals = _recurrence(dev, dtype, spec, len(name), shift)
    B, cuts, tail = 2, (70, 2, 3, 129), 5
    T = sum(cuts) + tail
    g = torch.Generator().manual_seed(11)
    proj = _rand(g, B, T, cols.total)
    want = [_recurrence_oracle(spec, cols, vals, proj[b]) for b in range(B)]
    p = proj.to(dev, dtype)
    br.alloc_state(B, T, dtype, dev)
    br.state.s.fill_(7.0)          # left over from someone else: a portion at position 0 starts anew
    br.state.conv.fill_(3.0)
    outs = []
    for plan in ((T,), cuts + (1,) * tail):
        out, at = [], 0
        for n in plan:
            pos = torch.tensor([at], device=dev) if (n == 1 and at > 0) else None
            out.append(br.heads(p[:, at:at + n], StepContext(None if pos is not None else at, pos, {})))
            at += n
        outs.append(torch.cat(out, 1).cpu())
        S = br.state.s.cpu()
        for b in range(B):
            assert hm.rms_error(S[b].flatten(1), want[b][1].flatten(1)) < (2e-5 if dtype == torch.float32 else 2e-2), (plan, b)
    w = torch.stack([x[0] for x in want])
    for got, plan in zip(outs, ("whole", "cut")):
        assert torch.isfinite(got.float()).all()
        # (z and the gate's product pass through the model's dtype in one of the two forms)
        assert hm.rms_error(got, w) < (5e-5 if dtype == torch.float32 else 4e-2), plan
    assert hm.rms_error(outs[1], outs[0].double()) < (5e-5 if dtype == torch.float32 else 3e-2)


def test_recurrence_segments_of_a_long_portion(dev, monkeypatch):
    from socket_amd import layer_ops
    from socket_amd.mixers import StepContext
    spec, _ = _specs()["delta"]
    br, cols, _ = _recurrence(dev, torch.float32, spec, 5)
    p = _rand(torch.Generator().manual_seed(1), 1, 300, cols.total).to(dev, torch.float32)
    br.alloc_state(1, 300, torch.float32, dev)
    one = br.heads(p, StepContext(0, None, {})).clone()
    s1 = br.state.s.clone()
    monkeypatch.setattr(layer_ops, "SCAN_SEGMENT", 128)
    many = br.heads(p, StepContext(0, None, {}))
    assert torch.allclose(one, many, atol=1e-5) and torch.allclose(s1, br.state.s, atol=1e-5)


# ---- whole models -------------------------------------------------------------------------------------

def _feed(model, tok, cuts, dev):
    """Logits [T,vocab] of one sequence (or [B,T,vocab] of a batch) fed in the given portions."""
    t = torch.tensor(tok, device=dev)
    t = t[None] if t.dim() == 1 else t
    out, at = [], 0
    for n in cuts:
        pos = torch.arange(at, at + n, device=dev)
        if n == 1 and at > 0:
            out.append(model(t[:, at:at + n], pos))
        else:
            out.append(model(t[:, at:at + n], pos, pos0=at, rows=range(n)))
        at += n
    y = torch.cat(out, 1).cpu()
    return y[0] if y.shape[0] == 1 else y


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("name", list(hm.CONFIGS))
def test_model_whole_portions_and_token_by_token(dev, tmp_path, dtype, name):
    cfg = hm.CONFIGS[name]
    w = hm.weights(cfg, seed=len(name))
    m = hm.build(tmp_path, cfg, w, dev, dtype)
    T = 90
    m.setup_caches(1, T)
    tok = hm.tokens(T, cfg["vocab"], 1)
    collect = []
    want = ho.forward(w, cfg, tok, collect)
    rng = random.Random(4)
    cuts = []
    while sum(cuts) < T:
        cuts.append(min(rng.choice([2, 3, 7, 24, 1]), T - sum(cuts)))
    for plan in ((T,), (1,) * T, tuple(cuts), (2,) * (T // 2), (T - 20,) + (1,) * 20):
        got = _feed(m, tok, plan, dev)
        assert hm.rms_error(got, want) < TOL[dtype], plan
        assert hm.mean_error(got, want) < MEAN_TOL[dtype], plan
    got = []
    m._run(torch.tensor([tok], device=dev), torch.arange(T, device=dev), False, 0, False, None, got)
    assert len(got) == len(collect)
    for a, b in zip(got, collect):
        assert hm.rms_error(a[0].cpu(), b) < TOL[dtype]


def test_model_batch_equals_each_alone_and_state_is_reused(dev, tmp_path):
    cfg = hm.CONFIGS["mixed"]
    w = hm.weights(cfg, seed=9, decay_shift=1.0)
    m = hm.build(tmp_path, cfg, w, dev, torch.float32)
    T = 60
    toks = [hm.tokens(T, cfg["vocab"], s) for s in (1, 2, 3, 4, 5)]     # (five rows: past the matrix-vector kernel)
    want = torch.stack([ho.forward(w, cfg, t) for t in toks])
    for cuts in ((T,), (31, 2, 3) + (1,) * 24):
        m.setup_caches(5, T)
        assert hm.rms_error(_feed(m, toks, cuts, dev), want) < TOL[torch.float32]
    # one state after another: a long request, a one-token one, a short one
    m.setup_caches(1, 200)
    for seed, n in ((6, 150), (7, 1), (8, 30), (6, 3)):
        tok = hm.tokens(n, cfg["vocab"], seed)
        cuts = (n - 2, 1, 1) if n > 3 else (n,)
        assert hm.rms_error(_feed(m, tok, cuts, dev), ho.forward(w, cfg, tok)) < TOL[torch.float32], n


def test_model_refuses_what_would_corrupt_its_state(dev, tmp_path):
    cfg = hm.CONFIGS["mixed"]
    m = hm.build(tmp_path, cfg, hm.weights(cfg), dev, torch.float32)
    m.setup_caches(1, 20)
    t = torch.tensor([[1, 2, 3]], device=dev)
    m(t, torch.arange(3, device=dev), pos0=0)
    with pytest.raises(RuntimeError, match="does not continue"):
        m(t, torch.arange(7, 10, device=dev), pos0=7)
    with pytest.raises(RuntimeError, match="out of bounds"):
        m(t, torch.arange(18, 21, device=dev), pos0=18)
    with pytest.raises(RuntimeError, match="sequences"):
        m(t.expand(2, 3), torch.arange(3, device=dev), pos0=0)
    with pytest.raises(ValueError, match="sparse"):
        m.sparse_forward(t, torch.arange(3, device=dev), pos0=0)


def _greedy(w, cfg, tok, n):
    tok = list(tok)
    margin = []
    for _ in range(n):
        lg = ho.forward(w, cfg, tok)[-1]
        top = torch.topk(lg, 2).values
        margin.append(float(top[0] - top[1]))
        tok.append(int(lg.argmax()))
    return tok, min(margin)


@pytest.mark.parametrize("graph,portion", [(True, 0), (False, 0), (True, 7)])
def test_greedy_generation(dev, tmp_path, graph, portion):
    """generate() with and without a recorded decode step, past several chunks, against the oracle's
    greedy continuation; the recorded step equals the eager one and leaves the state alone."""
    from socket_amd import generate as gen
    cfg = hm.CONFIGS["mixed"]
    w = hm.weights(cfg, seed=21)
    m = gen.load_model(hm.save(tmp_path, cfg, w), dev, torch.float32)
    prompt, n = hm.tokens(19, cfg["vocab"], 5), 40
    want, margin = _greedy(w, cfg, prompt, n)
    assert margin > 1e-4, "pick another seed: a near tie decides nothing"
    seq, st = gen.generate(m, torch.tensor([prompt, prompt], device=dev), n, decode_type="dense", use_graph=graph,
                           check_graph=graph, prefill_portion=portion)
    assert seq.tolist() == [want, want]
    if graph:
        assert st["graph_check"]["same_token"] and st["graph_check"]["max_abs_logit_diff"] < 1e-4


def test_command_line_generates_from_a_model_folder(dev, tmp_path):
    cfg = hm.CONFIGS["odd"]
    w = hm.weights(cfg, seed=2)
    path = hm.save(tmp_path, cfg, w)
    prompt = hm.tokens(9, cfg["vocab"], 5)
    want, margin = _greedy(w, cfg, prompt, 12)
    assert margin > 1e-4
    r = subprocess.run([sys.executable, "-m", "socket_amd.generate", "--model", path, "--dtype", "float32", "--prompt_tokens",
                        ",".join(map(str, prompt)), "--max_new_tokens", "12", "--print_tokens"], cwd=ROOT, capture_output=True,
                       text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert json.loads(r.stdout.splitlines()[-1])["dense"]["tokens"] == [want[9:]]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_run(dev, tmp_path, dtype):
    cfg = hm.CONFIGS["wide"]
    w = hm.weights(cfg, seed=4)
    path = hm.save(tmp_path / "m", cfg, w)
    out = tmp_path / "out"
    out.mkdir()
    steps, want = [], {}
    for name, n, cuts in (("a", 50, (30, 2, 1, 1, 16)), ("b", 1, (1,)), ("c", 45, (41, 1, 1, 1, 1))):
        tok = hm.tokens(n, cfg["vocab"], n)
        ref = ho.forward(w, cfg, tok)
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
                        "--max-tokens", "50"], input="\n".join(map(json.dumps, steps)) + "\n", capture_output=True, text=True,
                       timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [ln for ln in r.stdout.splitlines() if ln.startswith("done")] == [f"done {i}" for i in range(len(steps))]
    tol = TOL[getattr(torch, dtype)]
    for i in range(len(steps)):
        f = out / f"{i}.f32"
        assert f.exists() == (i in want)
        if i in want:
            got = torch.from_numpy(np.fromfile(f, dtype="<f4").reshape(want[i].shape))
            assert hm.rms_error(got, want[i]) < tol, i
