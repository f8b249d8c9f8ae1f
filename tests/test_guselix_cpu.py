"""Host side of the Guselix design: the config reader and loader, and what the oracle's own
definitions must satisfy (the chunked form of the generalized delta rule, absorbed latent
attention, averages over depth)."""
import copy
import math

import pytest
import torch

from oracle import guselix_oracle as go
from oracle import hybrid_oracle as ho
from tests import guselix_models as gm
from tests import hybrid_models as hm


def _shapes(w):
    return {k: tuple(v.shape) for k, v in w.items()}


def test_config_reader_takes_every_size_from_the_config():
    from socket_amd import guselix
    from socket_amd.mixers import LatentAttentionSpec
    cfg = gm.CONFIGS["odd"]
    a = guselix.args_from_config(cfg, _shapes(gm.weights(cfg, decay_rank=5)))
    assert (a.vocab_size, a.dim, a.norm_eps, a.n_layer, a.embed_scale) == (53, 37, 1e-4, 4, 1.0)
    assert a.tied_head and a.depth_average and not a.post_norm
    assert guselix.args_from_config(gm.CONFIGS["wide"], _shapes(gm.weights(gm.CONFIGS["wide"]))).embed_scale == 0.3
    d, l = a.layers[0].branches[0].spec, a.layers[1].branches[0].spec
    assert (d.heads, d.kv_heads, d.dim, d.vdim, d.decay_rank, d.removal, d.decay, d.q_scale, d.norm_per_head, d.taps) == \
        (2, 2, 10, 10, 5, True, "exp_sigmoid", 1.0, True, 0)
    assert d.decay_rate == math.exp(-0.5)
    assert l == LatentAttentionSpec(heads=5, dim=9, rot_dim=6, vdim=19, q_rank=13, kv_rank=11, rot_base=33.0, scale=0.4)
    assert (a.layers[0].mlp.ff, a.layers[0].mlp.bias, a.layers[0].mlp.act, a.layers[2].mlp) == (21, True, "silu", None)


@pytest.mark.parametrize("change", [
    lambda c: c["layers"][0].update(type="other"),
    lambda c: c["layers"][0]["mixer"].update(conv=3),
    lambda c: c["layers"][1]["mixer"].pop("scale"),
    lambda c: c["layers"][1]["mixer"]["rot"].update(dims=4),
    lambda c: c["layers"][1]["mixer"].update(mask={"size": 8}),
    lambda c: c["layers"][1]["mlp"].update(kind="sparse"),
    lambda c: c["embedding"].update(norm=True),
    lambda c: c.update(softcap=3.0),
])
def test_config_reader_refuses_what_it_does_not_know(change):
    from socket_amd import guselix
    cfg = copy.deepcopy(gm.CONFIGS["odd"])
    w = gm.weights(cfg)
    change(cfg)
    with pytest.raises(ValueError, match="config"):
        guselix.args_from_config(cfg, _shapes(w))


def test_loader_fills_every_parameter_and_reads_every_tensor(tmp_path):
    from socket_amd import registry
    cfg = gm.CONFIGS["mixed"]
    w = gm.weights(cfg, seed=3)
    m = registry.load_model(hm.save(tmp_path / "m", cfg, w), "cpu", torch.bfloat16)
    assert m.output is None and m.config.architecture == "Guselix"

    def column(lay, name):
        at = lay.columns.offset["0." + name]
        return lay.in_proj[at:at + lay.columns.rows["0." + name]].double()

    d = m.layers[1]
    for name, src in (("q", "r"), ("k", "k"), ("v", "v"), ("a1", "w1"), ("rate", "a"), ("g", "g")):
        assert torch.equal(column(d, name), w["l1.mix." + src]), name
    br = d.branches[0]
    assert torch.equal(br.rate_bias.double(), w["l1.mix.a.b"]) and torch.equal(br.decay_bias.double(), w["l1.mix.w0"])
    assert torch.equal(br.norm.double(), w["l1.mix.norm"]) and torch.equal(d.dwa.double(), w["l1.dwa"])
    assert all(t.dtype == torch.float32 for t in (br.rate_bias, br.decay_bias, br.norm, d.dwa, d.norm1, d.norm2))
    assert d.norm1b is None and torch.equal(d.gate_up_bias.double(), torch.cat([w["l1.mlp.gate.b"], w["l1.mlp.up.b"]]))
    assert torch.equal(d.down_bias.double(), w["l1.mlp.down.b"])
    a = m.layers[3]
    br = a.branches[0]
    assert torch.equal(torch.cat([column(a, "c"), column(a, "rot")]), w["l3.mix.dkv"]) and torch.equal(column(a, "cq"), w["l3.mix.dq"])
    assert torch.equal(br.uk.double(), w["l3.mix.uk"]) and torch.equal(br.uv.double(), w["l3.mix.uv"])
    assert br.q_norm.dtype == br.c_norm.dtype == torch.float32 and torch.equal(br.c_norm.double(), w["l3.mix.dkv.norm"])
    assert all(o % 8 == 0 for lay in m.layers for o in lay.columns.offset.values())
    for p in m.parameters():
        assert torch.isfinite(p.float()).all()
    # the norm of a feed-forward that is not there may be in the file, per-channel vectors may be [heads, dim]
    more = {**w, "l2.norm2": w["l2.norm1"], "l2.mix.w0": w["l2.mix.w0"].view(5, 24)}
    m2 = registry.load_model(hm.save(tmp_path / "more", cfg, more), "cpu", torch.float32)
    assert torch.equal(m2.layers[2].branches[0].decay_bias.double(), w["l2.mix.w0"])
    for bad, text in (({**w, "extra": w["embed"]}, "does not know"), ({k: v for k, v in w.items() if k != "l0.dwa"}, "no tensor"),
                      ({k: v for k, v in w.items() if k != "l1.mix.w1"}, "no tensor"), ({**w, "l0.dwa": w["l1.dwa"]}, "shape"),
                      ({**w, "l3.mix.dkv": w["l3.mix.dkv"][:-1]}, "shape")):
        with pytest.raises(ValueError, match=text):
            registry.load_model(hm.save(tmp_path / "bad", cfg, bad), "cpu", torch.bfloat16)


def test_recurrence_workspace_and_chunks_of_the_generalized_rule():
    from socket_amd import _lib
    if not __import__("os").path.exists(_lib.CORE_PATH):
        pytest.skip("libsocket_core.so is not built")
    L = _lib.core()
    assert [L.socket_recurrence_chunk(d, 1) for d in (16, 64, 65, 128, 256)] == [64, 64, 32, 32, 32]
    assert [L.socket_recurrence_chunk(d, 0) for d in (64, 128, 129)] == [64, 64, 32]
    plain, general = (L.socket_recurrence_workspace_bytes(1, 64, 1, 32, 32, r) for r in (0, 1))
    assert general - plain == 4 * (4 * 2 + 2 * 2) * 256     # read-out tiles and state tiles
    assert L.socket_recurrence_workspace_bytes(2, 65, 3, 32, 32, 1) == 2 * 3 * 2 * general


def test_general_delta_rule_removes_along_the_unit_key():
    """With no decay and rate one, a key written again replaces what the state held for it."""
    g = torch.Generator().manual_seed(0)
    k = torch.randn(1, 1, 8, generator=g, dtype=torch.float64)
    k = (k / k.norm()).expand(3, 1, 8)
    v = torch.randn(3, 1, 5, generator=g, dtype=torch.float64)
    one = torch.ones(3, 1, 8, dtype=torch.float64)
    o, S = go.general_delta_rule(k, k, v, one, one)
    assert torch.allclose(o, v, atol=1e-5) and torch.allclose(S[0].t() @ k[0, 0], v[-1, 0], atol=1e-5)
    # a longer key writes more but removes no more
    o2, _ = go.general_delta_rule(k, 2 * k, v, one, one)
    assert torch.allclose(o2, 2 * v, atol=1e-5)


def test_general_delta_rule_in_matrix_form_over_a_chunk():
    """The form the chunk kernels use: U = -Y from a triangular solve, read-outs and state from
    products with the state before the chunk."""
    g = torch.Generator().manual_seed(1)
    C, d, dv = 13, 6, 4
    r, k = (torch.randn(C, 1, d, generator=g, dtype=torch.float64) for _ in range(2))
    v = torch.randn(C, 1, dv, generator=g, dtype=torch.float64)
    w = go.decay_factor(torch.randn(C, 1, d, generator=g, dtype=torch.float64))
    a = ho.sigmoid(torch.randn(C, 1, d, generator=g, dtype=torch.float64))
    S0 = torch.randn(1, d, dv, generator=g, dtype=torch.float64)
    want, S1 = go.general_delta_rule(r, k, v, w, a, S0)
    r, k, v, w, a = (t[:, 0] for t in (r, k, v, w, a))
    n = ho.unit(k)
    b = torch.cumsum(torch.log(w), 0)
    bm = b - torch.log(w)
    Q, N, K, A = r * b.exp(), n * bm.exp(), k * (-b).exp(), a * n * (-b).exp()
    L, M = (N @ A.t()).tril(-1), (N @ K.t()).tril(-1)
    Y = torch.linalg.solve(torch.eye(C, dtype=torch.float64) + L, N @ S0[0] + M @ v)
    o = Q @ S0[0] + (Q @ K.t()).tril() @ v - (Q @ A.t()).tril() @ Y
    total = b[-1].exp()[:, None]
    S = total * (S0[0] + K.t() @ v - A.t() @ Y)
    assert torch.allclose(o, want[:, 0]) and torch.allclose(S, S1[0])


def test_general_delta_state_carries_over_a_cut():
    g = torch.Generator().manual_seed(2)
    x = [torch.randn(9, 2, 4, generator=g, dtype=torch.float64) for _ in range(5)]
    r, k, v, w, a = x[0], x[1], x[2], go.decay_factor(x[3]), ho.sigmoid(x[4])
    whole, S = go.general_delta_rule(r, k, v, w, a)
    o1, S1 = go.general_delta_rule(r[:4], k[:4], v[:4], w[:4], a[:4])
    o2, S2 = go.general_delta_rule(r[4:], k[4:], v[4:], w[4:], a[4:], S1)
    assert torch.equal(torch.cat([o1, o2]), whole) and torch.equal(S2, S)


def test_latent_attention_with_the_key_product_on_the_query_side():
    g = torch.Generator().manual_seed(3)
    T, H, dim, rot, rank, dv = 7, 3, 5, 4, 6, 8
    q = torch.randn(T, H, dim + rot, generator=g, dtype=torch.float64)
    c, kr = torch.randn(T, rank, generator=g, dtype=torch.float64), torch.randn(T, rot, generator=g, dtype=torch.float64)
    uk, uv = torch.randn(H * dim, rank, generator=g, dtype=torch.float64), torch.randn(H * dv, rank, generator=g, dtype=torch.float64)
    want = go.latent_attention(q, c, kr, uk, uv, H, dim, 0.3, 50.0)
    pos = torch.arange(T)
    ql = torch.stack([q[:, h, :dim] @ uk[h * dim:(h + 1) * dim] for h in range(H)], 1)
    qa = torch.cat([ql, ho.rotary(q[..., dim:], pos, rot, 50.0)], -1)
    key = torch.cat([c, ho.rotary(kr[:, None], pos, rot, 50.0)[:, 0]], -1)[:, None].expand(T, H, rank + rot)
    lat = go.causal_softmax_attention(qa, key, c[:, None].expand(T, H, rank), 0.3)
    got = torch.stack([lat[:, h] @ uv[h * dv:(h + 1) * dv].t() for h in range(H)], 1)
    assert torch.allclose(got, want)
    # the scale, the rotation of the shared part and causality each show
    assert not torch.allclose(go.latent_attention(q, c, kr, uk, uv, H, dim, 0.31, 50.0), want)
    assert not torch.allclose(go.latent_attention(q, c, kr, uk, uv, H, dim, 0.3, 60.0), want)
    c2 = c.clone()
    c2[-1] += 1
    assert torch.equal(go.latent_attention(q, c2, kr, uk, uv, H, dim, 0.3, 50.0)[:-1], want[:-1])


def test_layer_results_enter_the_average_before_their_own_averaging():
    cfg = gm.CONFIGS["mixed"]
    w = gm.weights(cfg, seed=5)
    tok = hm.tokens(6, cfg["vocab"], 1)
    col = []
    go.forward(w, cfg, tok, col)
    x0 = w["embed"][tok] * 2.5
    h = ho.rms_norm(x0, 1e-4, w["l0.norm1"])
    x1 = x0 + go.latent_mixer(w, "l0.mix", cfg["layers"][0]["mixer"], h, 1e-4)
    x1 = x1 + go.gated_feed_forward(w, "l0.mlp", ho.rms_norm(x1, 1e-4, w["l0.norm2"]))
    y1 = w["l0.dwa"][0] * x0 + w["l0.dwa"][1] * x1
    assert torch.allclose(col[0], y1)
    x2 = y1 + go.general_delta_mixer(w, "l1.mix", cfg["layers"][1]["mixer"], ho.rms_norm(y1, 1e-4, w["l1.norm1"]), 1e-4)
    x2 = x2 + go.gated_feed_forward(w, "l1.mlp", ho.rms_norm(x2, 1e-4, w["l1.norm2"]))
    assert torch.allclose(col[1], w["l1.dwa"][0] * x0 + w["l1.dwa"][1] * x1 + w["l1.dwa"][2] * x2)


def test_latent_cache_layout_and_splits():
    from socket_amd.layer_ops import latent_splits
    from socket_amd.sequence_state import LatentCache
    c = LatentCache(2, 10, 11, 6, torch.float32, "cpu")
    assert (c.rot_at, c.width, tuple(c.rows.shape), c.overwritten_by_a_step()) == (16, 24, (2, 10, 24), [])
    for cap in (1, 100, 5000, 10 ** 6):
        for tokens in (1, 5, 300):
            for heads in (1, 16, 130):
                n = latent_splits(cap, tokens, heads)
                assert 1 <= n <= 256 and (n == 1 or n * tokens * ((heads + 15) // 16) <= 256)


def test_rows_of_a_slice_are_evenly_spaced():
    from socket_amd.layer_ops import _row_stride
    x = torch.zeros(2, 3, 40)
    assert _row_stride(x) == 40 and _row_stride(x[..., 8:16]) == 40 and _row_stride(x[:, :1, 8:16]) == 120
    assert _row_stride(x[:1, :1, 8:16]) == 8
    with pytest.raises(AssertionError):
        _row_stride(x[:, :2, 8:16])


def test_bench_geometry():
    from socket_amd.workloads import guselix_args
    for size in ("2k", "4k"):
        g, m = guselix_args(size)
        assert g.architecture == "Guselix" and g.n_layer == m.n_layer and g.dim == m.dim
        assert {type(b.spec).__name__ for lay in g.layers for b in lay.branches} == {"LatentAttentionSpec", "RecurrenceSpec"}
        assert {lay.mlp.ff for lay in g.layers} == {lay.mlp.ff for lay in m.layers}
