"""Plain, slow implementation of the hybrid decoder (latent attention and channel-wise gated
delta-rule mixers, Dynamic Tanh norms): one function per mechanism, whole sequences, no cache,
no batching, no code shared with the package.  The tests compare the framework with it.

Weights are a dict name -> tensor under the checkpoint's names, the configuration is the
checkpoint's config.json as a dict.  Everything is computed in ``DT`` (float64 by default).
"""
from __future__ import annotations

import math

import torch

DT = torch.float64


# ------------------------------------------------------------------ mechanisms
def dynamic_tanh(x, w, b, alpha):
    """tanh(alpha x) w + b, elementwise: no statistics."""
    return torch.tanh(alpha * x) * w + b


def rms(x, eps):
    """x over its root mean square along the last axis, eps inside the root."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def silu(x):
    return x * torch.sigmoid(x)


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def rotate_interleaved(x, positions, base, dims):
    """x [T, ..., D]: the pairs (0, 1), (2, 3), ... of the first ``dims`` components of the
    last axis turned by position * base^(-2i / dims)."""
    out = x.clone()
    i = torch.arange(dims // 2, dtype=x.dtype)
    ang = positions.to(x.dtype)[:, None] * base ** (-2 * i / dims)
    shape = (x.shape[0],) + (1,) * (x.dim() - 2) + (dims // 2,)
    c, s = torch.cos(ang).reshape(shape), torch.sin(ang).reshape(shape)
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * c - v * s
    out[..., 1:dims:2] = v * c + u * s
    return out


def window_mask(n, size):
    """[n, n] bool, True where query i sees key j: itself and the size - 1 tokens before."""
    d = torch.arange(n)[:, None] - torch.arange(n)[None, :]
    ok = d >= 0
    return ok if size is None else ok & (d < size)


def sink_softmax(scores, ok, sink):
    """scores [H, n, n], sink [H] or None -> weights; the sink joins the denominator only."""
    sc = scores.masked_fill(~ok[None], float("-inf"))
    top = sc.max(-1, keepdim=True).values
    if sink is not None:
        top = torch.maximum(top, sink[:, None, None])
    e = torch.exp(sc - top)
    den = e.sum(-1, keepdim=True)
    if sink is not None:
        den = den + torch.exp(sink[:, None, None] - top)
    return e / den


def latent_attention(h, W, m, eps):
    """h [n, width] -> [n, width]; W: this mixer's tensors without their prefix."""
    n, H = h.shape[0], m["heads"]
    d, r, dv, R = m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos = torch.arange(n)
    q = (h @ W["q"].T).reshape(n, H, d + r)
    qn, qr = q[..., :d], rotate_interleaved(q[..., d:], pos, m["rot"]["base"], m["rot"]["dims"])
    kv = h @ W["dkv"].T
    c = rms(kv[:, :R], eps) * W["dkv.norm"]
    kr = rotate_interleaved(kv[:, R:], pos, m["rot"]["base"], m["rot"]["dims"])
    kn = (c @ W["uk"].T).reshape(n, H, d)
    v = (c @ W["uv"].T).reshape(n, H, dv)
    sc = (torch.einsum("ihd,jhd->hij", qn, kn) + torch.einsum("ihr,jr->hij", qr, kr)) * m["scale"]
    p = sink_softmax(sc, window_mask(n, m["mask"]["size"]), W["sink"])
    return torch.einsum("hij,jhv->ihv", p, v).reshape(n, H * dv) @ W["o"].T


def causal_conv(x, w):
    """x [n, C], w [C, taps]: the last tap is the current token's, zeros before the start."""
    taps = w.shape[1]
    pad = torch.cat([x.new_zeros(taps - 1, x.shape[1]), x])
    return sum(pad[j:j + x.shape[0]] * w[:, j] for j in range(taps))


def delta_scan(q, k, v, g, beta, S=None):
    """q, k, g [n, H, d], v [n, H, dv], beta [n, H] -> o [n, H, dv], S [H, d, dv]: decay the
    rows, correct what the key reads towards v, then read with q (after the write)."""
    n, H, d = k.shape
    S = q.new_zeros(H, d, v.shape[2]) if S is None else S.clone()
    out = torch.empty_like(v)
    for t in range(n):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - torch.einsum("hdv,hd->hv", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = torch.einsum("hdv,hd->hv", S, q[t])
    return out, S


def channel_delta(h, W, m, eps):
    n, H, Hk, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_conv(h @ W[x].T, W[x + ".conv"])) for x in "qkv")
    q = unit(q.reshape(n, Hk, d)) * d ** -0.5
    k = unit(k.reshape(n, Hk, d))
    of = torch.arange(H) // (H // Hk)
    beta = torch.sigmoid(h @ W["b"].T)
    raw = (h @ W["a1"].T) @ W["a2"].T + W["dt_bias"]
    step = torch.logaddexp(raw, torch.zeros_like(raw)).reshape(n, H, d)
    g = torch.exp(-torch.exp(W["A_log"])[None, :, None] * step)
    o, _ = delta_scan(q[:, of], k[:, of], v.reshape(n, H, dv), g, beta)
    gate = torch.sigmoid((h @ W["g1"].T) @ W["g2"].T).reshape(n, H, dv)
    return (rms(o, eps) * W["norm"] * gate).reshape(n, H * dv) @ W["o"].T


def gated_mlp(h, W):
    return (gelu_tanh(h @ W["gate"].T) * (h @ W["up"].T)) @ W["down"].T


# ------------------------------------------------------------------ the model
MIXERS = {"latent_attention": latent_attention, "channel_delta": channel_delta}


def forward(cfg, weights, tokens):
    """(logits [n, vocab], residual stream after every layer [layers, n, width])."""
    W = {k: (t if t.dtype == torch.int32 else t.to(DT)) for k, t in weights.items()}
    eps = cfg["norm"]["eps"]

    def norm(name, x):
        return dynamic_tanh(x, W[name], W[name + ".b"], W[name + ".alpha"])

    def sub(prefix):
        return {k[len(prefix):]: t for k, t in W.items() if k.startswith(prefix)}

    x = W["embed"][torch.as_tensor(list(tokens), dtype=torch.long)]
    stream = []
    for i, layer in enumerate(cfg["layers"]):
        x = x + MIXERS[layer["type"]](norm(f"l{i}.norm1", x), sub(f"l{i}.mix."), layer["mixer"], eps)
        if layer["mlp"] is not None:
            x = x + gated_mlp(norm(f"l{i}.norm2", x), sub(f"l{i}.mlp."))
        stream.append(x)
    return norm("final.norm", x) @ W["head"].T, torch.stack(stream)
