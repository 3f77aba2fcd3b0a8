"""Plain, slow implementation of the hybrid decoders: one function per mechanism, whole sequences,
no cache, no batching, no code shared with the package.  The tests compare the framework with it.

  Ralesun    latent attention and channel-wise gated delta-rule mixers, Dynamic Tanh norms
  Mebalorn   talking-heads attention and minGRU mixers beside a squared-relu feed-forward, layer
             norms, convolved sublayer inputs
  Nurilorn   attention with convolved projections, scaled rotation, capped scores, value mixing and
             head gates; clamped feed-forwards and routed experts, norms in groups, layer scales
  Garesun    retention, matrix memory (mLSTM) and latent attention whose latents several layers may
             share, beside squared-relu experts under one layer norm; per-layer token inputs

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


def latent_rows(h, W, m, eps):
    """What a token leaves for later ones: its normed latent, the rotated key part of all heads."""
    R = m["kv_rank"]
    kv = h @ W["dkv"].T
    return rms(kv[:, :R], eps) * W["dkv.norm"], \
        rotate_interleaved(kv[:, R:], torch.arange(h.shape[0]), m["rot"]["base"], m["rot"]["dims"])


def latent_read(h, W, m, rows, size, sink):
    """Every head's output [n, H, vdim] over ``rows``."""
    n, H = h.shape[0], m["heads"]
    d, r, dv = m["dim"], m["rot_dim"], m["vdim"]
    c, kr = rows
    q = (h @ W["q"].T).reshape(n, H, d + r)
    qn, qr = q[..., :d], rotate_interleaved(q[..., d:], torch.arange(n), m["rot"]["base"], m["rot"]["dims"])
    kn = (c @ W["uk"].T).reshape(n, H, d)
    v = (c @ W["uv"].T).reshape(n, H, dv)
    sc = (torch.einsum("ihd,jhd->hij", qn, kn) + torch.einsum("ihr,jr->hij", qr, kr)) * m["scale"]
    p = sink_softmax(sc, window_mask(n, size), sink)
    return torch.einsum("hij,jhv->ihv", p, v)


def latent_attention(h, W, m, eps):
    """h [n, width] -> [n, width]; W: this mixer's tensors without their prefix."""
    o = latent_read(h, W, m, latent_rows(h, W, m, eps), m["mask"]["size"], W["sink"])
    return o.flatten(1) @ W["o"].T


def gated_latent_attention(h, W, m, eps, held):
    """Without window and sink, a sigmoid gate per head; ``held``: another layer's rows, or None."""
    rows = latent_rows(h, W, m, eps) if held is None else held
    o = latent_read(h, W, m, rows, None, None) * torch.sigmoid(h @ W["g"].T)[:, :, None]
    return o.flatten(1) @ W["o"].T, rows


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


def sinusoids(n, width):
    """[n, width]: entry 2i is sin(p base^(-2i / width)), entry 2i + 1 the cosine."""
    out = torch.zeros(n, width, dtype=DT)
    for c in range(width):
        ang = torch.arange(n, dtype=DT) * 10000.0 ** (-2 * (c // 2) / width)
        out[:, c] = torch.cos(ang) if c % 2 else torch.sin(ang)
    return out


def layer_norm(x, w, b, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w + b


def convolved(h, w):
    """A sublayer's input with a causal convolution over time added, channel by channel."""
    return h + causal_conv(h, w)


def talking_attention(h, W, m, eps):
    """Grouped-query attention without rotation; unit-rms queries and keys; a softmax sink per
    head; the normalised weights of all heads mixed by ``talk`` before they meet the values."""
    n, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms((h @ W["q"].T + W["q.b"]).reshape(n, H, d), eps) * W["q.norm"]
    k = rms((h @ W["k"].T + W["k.b"]).reshape(n, G, d), eps) * W["k.norm"]
    v = (h @ W["v"].T + W["v.b"]).reshape(n, G, dv)
    of = torch.arange(H) // (H // G)
    sc = torch.einsum("ihd,jhd->hij", q, k[:, of]) * m["scale"]
    p = sink_softmax(sc, window_mask(n, None), W["sink"])
    p = torch.einsum("hg,gij->hij", W["talk"], p)
    return torch.einsum("hij,jhv->ihv", p, v[:, of]).reshape(n, H * dv) @ W["o"].T


def gated_average(z, u, S=None):
    """S_t = (1 - z_t) S_(t-1) + z_t c_t with c = u + 1/2 where u >= 0, else sigmoid(u);
    z, u [n, C] -> every S_t."""
    S = z.new_zeros(z.shape[1]) if S is None else S
    out = []
    for t in range(z.shape[0]):
        c = torch.where(u[t] >= 0, u[t] + 0.5, torch.sigmoid(u[t]))
        S = (1 - z[t]) * S + z[t] * c
        out.append(S)
    return torch.stack(out)


def mingru(h, W, m, eps):
    S = gated_average(torch.sigmoid(h @ W["z"].T + W["z.b"]), h @ W["x"].T + W["x.b"])
    return (S * silu(h @ W["g"].T)) @ W["o"].T


def relu2_mlp(h, W):
    return torch.relu(h @ W["up"].T).square() @ W["down"].T


def group_rms(x, w, groups, eps):
    """Each of ``groups`` equal consecutive parts over its own root mean square, then w."""
    parts = x.reshape(*x.shape[:-1], groups, -1)
    return rms(parts, eps).reshape(x.shape) * w


def scaled_rotation(dims, base, scaling):
    """(turns' speeds [dims / 2], factor of cosine and sine): fast pairs keep base^(-2i / dims), slow
    ones are divided by ``factor``, a ramp between the pairs that turn ``fast`` and ``slow`` times
    within ``original`` positions."""
    f = base ** (-2 * torch.arange(dims // 2, dtype=DT) / dims)
    if not scaling:
        return f, 1.0
    def pair(turns):
        return dims * math.log(scaling["original"] / (2 * math.pi * turns)) / (2 * math.log(base))
    lo, hi = max(math.floor(pair(scaling["fast"])), 0), min(math.ceil(pair(scaling["slow"])), dims - 1)
    ramp = ((torch.arange(dims // 2, dtype=DT) - lo) / max(hi - lo, 0.001)).clamp(0, 1)
    return f / scaling["factor"] * ramp + f * (1 - ramp), 0.1 * math.log(scaling["factor"]) + 1


def rotate_scaled(x, positions, rot):
    """x [T, heads, D]: interleaved pairs of the first rot.dims components."""
    f, mag = scaled_rotation(rot["dims"], rot["base"], rot.get("scaling"))
    a = positions.to(x.dtype)[:, None, None] * f
    c, s = torch.cos(a) * mag, torch.sin(a) * mag
    out = x.clone()
    u, v = x[..., 0:rot["dims"]:2], x[..., 1:rot["dims"]:2]
    out[..., 0:rot["dims"]:2] = u * c - v * s
    out[..., 1:rot["dims"]:2] = v * c + u * s
    return out


def zero_sink_softmax(scores, ok):
    """exp(s) / (1 + sum exp(s)) over the last axis: a sink of score 0 without a value."""
    sc = scores.masked_fill(~ok, float("-inf"))
    top = sc.max(-1, keepdim=True).values.clamp(min=0)
    e = torch.exp(sc - top)
    return e / (torch.exp(-top) + e.sum(-1, keepdim=True))


def mixed_values(v, first, lam):
    """(1 - lam) v + lam first."""
    return (1 - lam) * v + lam * first


def capped_attention(h, W, m, v_first):
    """-> (output [n, width], this layer's values before any mixing)."""
    n, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (causal_conv(h @ W[x].T, W[x + ".conv"]) if m["conv"] else h @ W[x].T for x in "qkv")
    pos = torch.arange(n)
    q = rotate_scaled(q.reshape(n, H, d), pos, m["rot"])
    k = rotate_scaled(k.reshape(n, G, d), pos, m["rot"])
    own = v
    if m["v_mix"] and v_first is not None:
        v = mixed_values(v, v_first, W["vmix"])
    v = v.reshape(n, G, dv)
    of = torch.arange(H) // (H // G)
    sc = torch.einsum("ihd,jhd->hij", q, k[:, of]) * m["scale"]
    if m["softcap"]:
        sc = m["softcap"] * torch.tanh(sc / m["softcap"])
    p = zero_sink_softmax(sc, window_mask(n, None))
    o = torch.einsum("hij,jhv->ihv", p, v[:, of])
    o = o * torch.sigmoid(h @ W["g"].T)[:, :, None]
    return o.reshape(n, H * dv) @ W["o"].T, own


def clamped_mlp(h, W, limit, prefix=""):
    g = (h @ W[prefix + "gate"].T).clamp(max=limit)
    u = (h @ W[prefix + "up"].T).clamp(-limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1)) @ W[prefix + "down"].T


def route(h, w, r):
    """[n, experts] weights, zero where a token does not go: softmax scores, the best groups by
    their best expert, the best experts in them, divided by their sum."""
    s = torch.softmax(h @ w.T, -1)
    n, E = s.shape
    groups = r.get("groups") or {"count": 1, "keep": 1}
    best = s.reshape(n, groups["count"], -1).max(-1).values
    keep = torch.zeros_like(best).scatter(1, best.topk(groups["keep"], -1).indices, 1.0)
    open_ = keep.repeat_interleave(E // groups["count"], 1) > 0
    top = s.masked_fill(~open_, -1.0).topk(r["top"], -1).indices
    w = torch.zeros_like(s).scatter(1, top, s.gather(1, top))
    return w / (w.sum(-1, keepdim=True) + 1e-20)


def route_margin(h, w, r):
    """[n] how far the closest call of each token's choice is, in logits: between the last group
    kept and the next, the last expert chosen and the next in those groups."""
    z = h @ w.T
    n, E = z.shape
    groups = r.get("groups") or {"count": 1, "keep": 1}
    best = z.reshape(n, groups["count"], -1).max(-1).values.sort(-1, descending=True)
    keep, out = groups["keep"], torch.full((n,), math.inf, dtype=z.dtype)
    if keep < groups["count"]:
        out = best.values[:, keep - 1] - best.values[:, keep]
    open_ = torch.zeros(n, groups["count"], dtype=torch.bool).scatter(1, best.indices[:, :keep], True)
    z = z.masked_fill(~open_.repeat_interleave(E // groups["count"], 1), -math.inf).sort(-1, descending=True).values
    return torch.minimum(out, z[:, r["top"] - 1] - z[:, r["top"]]) if r["top"] < E else out


def experts(h, W, mlp):
    w = route(h, W["router"], mlp["router"])
    return sum(w[:, e:e + 1] * clamped_mlp(h, W, mlp["expert"]["limit"], f"e{e}.")
               for e in range(w.shape[1]))


def rotate_halves(x, positions, base, dims):
    """x [T, heads, D]: components i and i + dims / 2 turned by position * base^(-2i / dims)."""
    half = dims // 2
    i = torch.arange(half, dtype=x.dtype)
    a = positions.to(x.dtype)[:, None, None] * base ** (-2 * i / max(dims, 1))
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * torch.cos(a) - v * torch.sin(a), v * torch.cos(a) + u * torch.sin(a), x[..., dims:]], -1)


def retention_scan(q, k, v, decay, S=None):
    """S <- decay S + k v^T, o = S^T q; q, k [n, H, d], v [n, H, dv], decay [H]."""
    S = q.new_zeros(q.shape[1], q.shape[2], v.shape[2]) if S is None else S
    out = []
    for t in range(q.shape[0]):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out.append(torch.einsum("hdv,hd->hv", S, q[t]))
    return torch.stack(out), S


def retention(h, W, m, eps):
    n, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    pos, rot = torch.arange(n), m.get("rot") or {"base": 1.0, "dims": 0}
    q = rotate_halves((h @ W["q"].T).reshape(n, H, d), pos, rot["base"], rot["dims"])
    k = rotate_halves((h @ W["k"].T).reshape(n, H, d), pos, rot["base"], rot["dims"]) * d ** -0.5
    o, _ = retention_scan(q, k, (h @ W["v"].T).reshape(n, H, dv), torch.tensor(m["decay"], dtype=h.dtype))
    return (rms(o, eps).reshape(n, H * dv) * silu(h @ W["g"].T)) @ W["o"].T


def memory_scan(q, k, v, i, f, state=None):
    """Matrix memory with log gates i, f [n, H] and a running maximum from 0 -> every read-out, the
    state (S, normaliser, maximum)."""
    H, d, dv = q.shape[1], q.shape[2], v.shape[2]
    S, N, top = state or (q.new_zeros(H, d, dv), q.new_zeros(H, d), q.new_zeros(H))
    out = []
    for t in range(q.shape[0]):
        new = torch.maximum(f[t] + top, i[t])
        keep, put = torch.exp(f[t] + top - new), torch.exp(i[t] - new)
        S = keep[:, None, None] * S + put[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        N = keep[:, None] * N + put[:, None] * k[t]
        top = new
        den = torch.maximum((N * q[t]).sum(-1).abs(), torch.exp(-top)) + 1e-6
        out.append(torch.einsum("hdv,hd->hv", S, q[t]) / den[:, None])
    return torch.stack(out), (S, N, top)


def memory_gates(h, W, cap):
    """Log input gate, log forget gate."""
    i, f = (cap * torch.tanh((h @ W[x].T + W[x + ".b"]) / cap) for x in "if")
    return i, -torch.logaddexp(-f, torch.zeros_like(f))


def mlstm(h, W, m, eps):
    n, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ W["q"].T).reshape(n, H, d) * d ** -0.5
    o, _ = memory_scan(q, (h @ W["k"].T).reshape(n, H, d), (h @ W["v"].T).reshape(n, H, dv),
                       *memory_gates(h, W, m["gate_cap"]))
    return (rms(o, eps).reshape(n, H * dv) * W["norm"] * torch.sigmoid(h @ W["g"].T)) @ W["o"].T


def relu2_experts(h, W, mlp):
    """Squared-relu experts: softmax over the chosen logits; a shared one for every token."""
    z = h @ W["router"].T
    top = z.topk(mlp["router"]["top"], -1)
    w = torch.zeros_like(z).scatter(1, top.indices, torch.softmax(top.values, -1))

    def sub(p):
        return {x: W[p + x] for x in ("up", "down")}

    y = sum(w[:, e:e + 1] * relu2_mlp(h, sub(f"e{e}.")) for e in range(z.shape[1]))
    return y + relu2_mlp(h, sub("shared.")) if mlp.get("shared") else y


def token_side(x, e, W, eps):
    """A token's own input to a layer, gated by the stream: what is added to it."""
    y = (gelu_tanh(x @ W["gate"].T) * e) @ W["proj"].T
    return rms(y, eps) * W["norm"]


# ------------------------------------------------------------------ the models
MIXERS = {"latent_attention": latent_attention, "channel_delta": channel_delta,
          "attention": talking_attention, "mingru": mingru}


def forward(cfg, weights, tokens, margins=None):
    """(logits [n, vocab], residual stream after every layer [layers, n, width]).  ``margins``: a
    list that takes every routed layer's ``route_margin``."""
    if cfg["architecture"] == "Nurilorn":
        return _nurilorn(cfg, weights, tokens, margins)
    if cfg["architecture"] == "Garesun":
        return _garesun(cfg, weights, tokens, margins)
    return {"Ralesun": _ralesun, "Mebalorn": _mebalorn}[cfg["architecture"]](cfg, weights, tokens)


def _nurilorn(cfg, weights, tokens, margins=None):
    W = {k: t.to(DT) for k, t in weights.items()}
    mult = cfg["residual_mult"]

    def norm(name, x):
        return group_rms(x, W[name], cfg["norm"]["groups"], cfg["norm"]["eps"])

    def sub(prefix):
        return {k[len(prefix):]: t for k, t in W.items() if k.startswith(prefix)}

    x = W["embed"][torch.as_tensor(list(tokens), dtype=torch.long)] * cfg["embedding"]["scale"]
    stream, v_first = [], None
    for i, layer in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", layer["mixer"], layer["mlp"]
        y, v = capped_attention(norm(p + "norm1", x), sub(p + "mix."), m, v_first)
        if m["v_mix"] and v_first is None:
            v_first = v
        x = x + mult * (y * W[p + "ls1"])
        if mlp is not None:
            h = norm(p + "norm2", x)
            if margins is not None and mlp["kind"] == "moe":
                margins.append(route_margin(h, W[p + "mlp.router"], mlp["router"]))
            y = clamped_mlp(h, sub(p + "mlp."), mlp["limit"]) if mlp["kind"] == "dense" else \
                experts(h, sub(p + "mlp."), mlp)
            x = x + mult * (y * W[p + "ls2"])
        stream.append(x)
    return norm("final.norm", x) @ W["head"].T * cfg["logit_scale"], torch.stack(stream)


def _garesun(cfg, weights, tokens, margins=None):
    W = {k: t.to(DT) for k, t in weights.items()}
    eps, dim = cfg["norm"]["eps"], cfg["token_side"]["dim"]
    toks = torch.as_tensor(list(tokens), dtype=torch.long)

    def sub(prefix):
        return {k[len(prefix):]: t for k, t in W.items() if k.startswith(prefix)}

    x = W["embed"][toks] * cfg["embedding"]["scale"]
    stream, rows = [], {}
    for i, layer in enumerate(cfg["layers"]):
        m, mix = layer["mixer"], sub(f"l{i}.mix.")
        h = layer_norm(x, W[f"l{i}.norm1"], 0.0, eps)
        if layer["type"] == "latent_attention":
            y, rows[i] = gated_latent_attention(h, mix, m, eps, rows.get(m.get("kv_from")))
        else:
            y = {"retention": retention, "mlstm": mlstm}[layer["type"]](h, mix, m, eps)
        if layer["mlp"] is not None:
            if margins is not None:
                margins.append(route_margin(h, W[f"l{i}.mlp.router"], layer["mlp"]["router"]))
            y = y + relu2_experts(h, sub(f"l{i}.mlp."), layer["mlp"])
        x = x + y
        x = x + token_side(x, W["side.embed"][toks, i * dim:(i + 1) * dim], sub(f"l{i}.side."), eps)
        stream.append(x)
    return layer_norm(x, W["final.norm"], 0.0, eps) @ W["head"].T, torch.stack(stream)


def _mebalorn(cfg, weights, tokens):
    W = {k: t.to(DT) for k, t in weights.items()}
    eps, cap = cfg["norm"]["eps"], cfg["logit_softcap"]

    def sub(prefix):
        return {k[len(prefix):]: t for k, t in W.items() if k.startswith(prefix)}

    x = W["embed"][torch.as_tensor(list(tokens), dtype=torch.long)]
    x = x + sinusoids(len(tokens), cfg["width"])
    stream = []
    for i, layer in enumerate(cfg["layers"]):
        def read(k):
            n = f"l{i}.norm{k}"
            return convolved(layer_norm(x, W[n], W[n + ".b"], eps), W[f"l{i}.canon{k}"])

        y = MIXERS[layer["type"]](read(1), sub(f"l{i}.mix."), layer["mixer"], eps)
        if layer["mlp"] is not None:
            y = y + relu2_mlp(read(2), sub(f"l{i}.mlp."))
        x = x + y
        stream.append(x)
    lg = layer_norm(x, W["final.norm"], W["final.norm.b"], eps) @ W["head"].T
    return cap * torch.tanh(lg / cap), torch.stack(stream)


def _ralesun(cfg, weights, tokens):
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
