"""Small Guselix configurations with random weights for the tests: config dicts and weights
under the checkpoint's names (bf16-representable values)."""
from __future__ import annotations

import math

import torch


def delta(heads=3, dim=16):
    return {"heads": heads, "dim": dim}


def latent(heads=3, dim=16, rot_dim=8, vdim=24, q_rank=40, kv_rank=32, base=700.0, scale=None):
    return {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
            "rot": {"base": base, "dims": rot_dim}, "scale": (dim + rot_dim) ** -0.5 if scale is None else scale}


def mlp(ff=56):
    return {"kind": "dense", "ff": ff}


def delta_layer(mixer=None, ff=None):
    return {"type": "general_delta", "mixer": mixer or delta(), "mlp": ff}


def latent_layer(mixer=None, ff=None):
    return {"type": "latent_attention", "mixer": mixer or latent(), "mlp": ff}


def config(layers, width=48, vocab=91, eps=1e-4, scale=2.5):
    return {"architecture": "Guselix", "embedding": {"scale": scale}, "layers": layers, "norm": {"eps": eps}, "vocab": vocab,
            "width": width}


CONFIGS = {
    # both mixers with and without a feed-forward, attention first, in the middle and last
    "mixed": config([latent_layer(ff=mlp()), delta_layer(ff=mlp(40)), delta_layer(delta(5, 24)),
                     latent_layer(latent(2, 40, 16, 8, 24, 72, 90.0, 0.21)), delta_layer(delta(1, 64), mlp(24)), latent_layer()]),
    # nothing is a multiple of eight (scalar paths), a value width above the key's, one head
    "odd": config([delta_layer(delta(2, 10), mlp(21)), latent_layer(latent(5, 9, 6, 19, 13, 11, 33.0, 0.4), mlp(33)),
                   latent_layer(latent(1, 3, 2, 1, 5, 7, 3.0, 1.0)), delta_layer(delta(3, 7))], width=37, vocab=53, scale=1.0),
    # wider heads (32-token chunks of the recurrence, other sizes of the matrix-core kernels), more heads than a tile
    "wide": config([delta_layer(delta(1, 136)), latent_layer(latent(18, 96, 32, 64, 64, 136, 2000.0), mlp(72)),
                    delta_layer(delta(2, 80), mlp(64)), latent_layer(latent(2, 128, 64, 128, 128, 320, 9000.0))], width=64, vocab=120,
                   eps=1e-6, scale=0.3),
}


def weights(cfg, seed=0, decay_rank=12, decay_shift=0.0):
    """float64 tensors whose values are exact in bf16.  decay_shift > 0: stronger decays."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]

    def rand(*shape):
        return torch.randn(*shape, generator=g, dtype=torch.float64)

    def mat(n, k, gain=1.0):
        return rand(n, k) * gain / math.sqrt(k)

    def norm(n):
        return 1.0 + 0.3 * rand(n)

    w = {"embed": rand(V, W), "final.norm": norm(W)}
    for i, lay in enumerate(cfg["layers"]):
        p, c = f"l{i}.", lay["mixer"]
        m = p + "mix"
        w[p + "norm1"] = norm(W)
        # (unequal weights of either sign, so that no result can stand in for another)
        w[p + "dwa"] = 0.4 * rand(i + 2) + torch.cat([torch.zeros(i + 1, dtype=torch.float64), torch.ones(1, dtype=torch.float64)])
        if lay["type"] == "general_delta":
            n = c["heads"] * c["dim"]
            for t in "rkvag":
                w[f"{m}.{t}"] = mat(n, W, 1.0 if t != "k" else 1.0 / math.sqrt(c["dim"]))
            w[m + ".a.b"] = rand(n)
            w[m + ".w1"], w[m + ".w2"] = mat(decay_rank, W, 1.5), mat(n, decay_rank, 1.5)
            w[m + ".w0"] = 2 * rand(n) - 2.0 + decay_shift
            w[m + ".norm"], w[m + ".o"] = norm(n), mat(W, n)
        else:
            H, d, r, dv = c["heads"], c["dim"], c["rot_dim"], c["vdim"]
            w[m + ".dq"], w[m + ".dq.norm"] = mat(c["q_rank"], W), norm(c["q_rank"])
            w[m + ".uq"] = mat(H * (d + r), c["q_rank"], 2.0)       # (scores that pick among the keys)
            w[m + ".dkv"], w[m + ".dkv.norm"] = mat(c["kv_rank"] + r, W), norm(c["kv_rank"])
            w[m + ".uk"], w[m + ".uv"] = mat(H * d, c["kv_rank"]), mat(H * dv, c["kv_rank"])
            w[m + ".g"], w[m + ".o"] = mat(H * dv, W), mat(W, H * dv)
        if lay["mlp"]:
            ff = lay["mlp"]["ff"]
            w[p + "norm2"] = norm(W)
            for t, a, b in (("gate", ff, W), ("up", ff, W), ("down", W, ff)):
                w[f"{p}mlp.{t}"], w[f"{p}mlp.{t}.b"] = mat(a, b), 0.5 * rand(a)
    return {k: v.to(torch.bfloat16).double() for k, v in w.items()}
