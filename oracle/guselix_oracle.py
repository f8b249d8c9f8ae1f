"""Plain restatement of the Guselix decoder in torch float64 (or any dtype): one function
per mechanism, token by token where the definition is a recurrence.  Test
infrastructure: no cache, nothing fused, no code shared with socket_amd.

`weights` is a flat dict of tensors under the checkpoint's names, `cfg` the parsed
config.json.  Everything is computed in the dtype the weights have.
"""
from __future__ import annotations

import math

import torch

from .hybrid_oracle import linear, rms_norm, rotary, sigmoid, silu, unit

DECAY_RATE = math.exp(-0.5)


def decay_factor(z, rate=DECAY_RATE):
    """Between exp(-rate) (z large) and 1."""
    return torch.exp(-rate * sigmoid(z))


def general_delta_rule(r, k, v, w, a, state=None):
    """r, k [T,H,dk], v [T,H,dv], w (decay factors) and a (removal rates) [T,H,dk].  With u the
    unit vector of k and S the state before the token: what S holds for u is removed along
    a * u, S decays per key channel, k v^T is added; the output reads the new state with r.
    Returns outputs [T,H,dv] and the final state [H,dk,dv]."""
    T, H, dk = r.shape
    S = r.new_zeros(H, dk, v.shape[-1]) if state is None else state.clone()
    u = unit(k)
    out = []
    for t in range(T):
        held = (S * u[t][:, :, None]).sum(1)                        # [H,dv], of the old state
        S = (S * w[t][:, :, None] - (a[t] * u[t])[:, :, None] * held[:, None, :]
             + k[t][:, :, None] * v[t][:, None, :])
        out.append((S * r[t][:, :, None]).sum(1))
    return torch.stack(out), S


def general_delta_mixer(w, pre, c, h, eps):
    T = h.shape[0]
    H, d = c["heads"], c["dim"]
    r, k, v = (linear(w[pre + n], h).view(T, H, d) for n in (".r", ".k", ".v"))
    z = linear(w[pre + ".w2"], torch.tanh(linear(w[pre + ".w1"], h))) + w[pre + ".w0"].reshape(-1)
    a = sigmoid(linear(w[pre + ".a"], h) + w[pre + ".a.b"].reshape(-1))
    o, _ = general_delta_rule(r, k, v, decay_factor(z).view(T, H, d), a.view(T, H, d))
    o = rms_norm(o, eps).reshape(T, H * d) * w[pre + ".norm"].reshape(-1)
    return linear(w[pre + ".o"], o * sigmoid(linear(w[pre + ".g"], h)))


def causal_softmax_attention(q, k, v, scale):
    """q, k [T,H,d], v [T,H,dv]; position i sees every j <= i."""
    T = q.shape[0]
    out = q.new_zeros(T, q.shape[1], v.shape[-1])
    for h in range(q.shape[1]):
        s = (q[:, h] @ k[:, h].t()) * scale
        s = s.masked_fill(torch.ones(T, T, dtype=torch.bool).triu(1), -math.inf)
        p = torch.exp(s - s.max(-1, keepdim=True).values)
        out[:, h] = (p / p.sum(-1, keepdim=True)) @ v[:, h]
    return out


def latent_attention(q, latent, k_rot, w_uk, w_uv, heads, dim, scale, rot_base):
    """q [T,heads,dim + rot] (rotated part last, not yet turned), latent [T,kv_rank], k_rot
    [T,rot] (not yet turned), w_uk [heads*dim,kv_rank], w_uv [heads*vdim,kv_rank]."""
    T, rot = k_rot.shape
    pos = torch.arange(T)
    k = linear(w_uk, latent).view(T, heads, dim)
    v = linear(w_uv, latent).view(T, heads, -1)
    kr = rotary(k_rot[:, None], pos, rot, rot_base).expand(T, heads, rot)
    qr = rotary(q[..., dim:], pos, rot, rot_base)
    return causal_softmax_attention(torch.cat([q[..., :dim], qr], -1), torch.cat([k, kr], -1), v, scale)


def latent_mixer(w, pre, c, h, eps):
    T = h.shape[0]
    H, dim, rot, rank = c["heads"], c["dim"], c["rot_dim"], c["kv_rank"]
    cq = rms_norm(linear(w[pre + ".dq"], h), eps, w[pre + ".dq.norm"])
    q = linear(w[pre + ".uq"], cq).view(T, H, dim + rot)
    down = linear(w[pre + ".dkv"], h)
    latent = rms_norm(down[:, :rank], eps, w[pre + ".dkv.norm"])
    o = latent_attention(q, latent, down[:, rank:], w[pre + ".uk"], w[pre + ".uv"], H, dim, c["scale"], c["rot"]["base"])
    return linear(w[pre + ".o"], o.reshape(T, -1) * sigmoid(linear(w[pre + ".g"], h)))


def gated_feed_forward(w, pre, h):
    g = linear(w[pre + ".gate"], h) + w[pre + ".gate.b"]
    u = linear(w[pre + ".up"], h) + w[pre + ".up.b"]
    return linear(w[pre + ".down"], silu(g) * u) + w[pre + ".down.b"]


def depth_average(results, weights):
    """Sum of weights[j] * results[j]: the embedding output and every layer's result so far."""
    return sum(weights[j] * x for j, x in enumerate(results))


MIXERS = {"general_delta": general_delta_mixer, "latent_attention": latent_mixer}


def forward(weights, cfg, tokens, collect=None):
    """tokens: list of ints -> logits [T,vocab]; `collect` (a list) receives the stream after
    every layer."""
    w, eps = weights, cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
    results = [x]
    for i, layer in enumerate(cfg["layers"]):
        pre = f"l{i}"
        x = x + MIXERS[layer["type"]](w, pre + ".mix", layer["mixer"], rms_norm(x, eps, w[pre + ".norm1"]), eps)
        if layer["mlp"] is not None:
            x = x + gated_feed_forward(w, pre + ".mlp", rms_norm(x, eps, w[pre + ".norm2"]))
        results.append(x)
        x = depth_average(results, w[pre + ".dwa"])
        if collect is not None:
            collect.append(x.clone())
    return linear(w["embed"], rms_norm(x, eps, w["final.norm"]))
