"""Small random models of mixed layer kinds for the tests: configuration dicts in the
checkpoint's format, weights under its names, checkpoint folders, and error measures."""
from __future__ import annotations

import json
import os
import struct

import torch


def latent(heads, dim, rot, vdim, rank, window, base=10000.0, scale=None, ff=None):
    return {"type": "latent_attention", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank,
                      "scale": scale or (dim + rot) ** -0.5, "mask": {"size": window},
                      "rot": {"base": base, "dims": rot}}}


def delta(heads, kv_heads, dim, vdim, taps, ff=None):
    return {"type": "channel_delta", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": taps}}


def attention(heads, kv_heads, dim, vdim, scale=None, ff=None):
    return {"type": "attention", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                      "scale": scale or dim ** -0.5}}


def mingru(width, ff=None):
    return {"type": "mingru", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"width": width}}


def grouped(heads, kv_heads, dim, vdim, rot, conv=3, base=10000.0, scaling=None, cap=20.0, v_mix=True,
            scale=None, ff=None, experts=None, top=2, groups=None, limit=1.5):
    """``scaling``: (factor, original, fast, slow); ``groups``: (count, keep)."""
    if experts:
        router = {"experts": experts, "top": top}
        if groups:
            router["groups"] = {"count": groups[0], "keep": groups[1]}
        mlp = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": router}
    else:
        mlp = {"kind": "dense", "ff": ff, "limit": limit} if ff else None
    rot = {"base": base, "dims": rot}
    if scaling:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "rot": rot,
                      "scale": scale or dim ** -0.5, "softcap": cap, "v_mix": v_mix}}


def scaled(vocab, width, *layers, eps=1e-5, groups=2, embed=3.0, mult=0.8, logits=1.5):
    return {"architecture": "Nurilorn", "vocab": vocab, "width": width, "norm": {"eps": eps, "groups": groups},
            "embedding": {"scale": embed}, "residual_mult": mult, "logit_scale": logits, "layers": list(layers)}


def _moe(ff, experts, top, shared):
    if not ff:
        return None
    out = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    return {**out, "shared": {"ff": shared}} if shared else out


def retention(heads, dim, vdim, rot=0, decay=None, base=10000.0, ff=None, experts=6, top=2, shared=None):
    decay = decay or [1 - 2.0 ** (-1 - 7 * h / heads) for h in range(heads)]
    return {"type": "retention", "mlp": _moe(ff, experts, top, shared),
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay, "rot": {"base": base, "dims": rot}}}


def mlstm(heads, dim, vdim, cap=9.0, ff=None, experts=6, top=2, shared=None):
    return {"type": "mlstm", "mlp": _moe(ff, experts, top, shared),
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}}


def gated_latent(heads, dim, rot, vdim, rank, kv_from=None, base=10000.0, scale=None, ff=None, experts=6, top=2,
                 shared=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank,
         "scale": scale or (dim + rot) ** -0.5, "rot": {"base": base, "dims": rot}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mlp": _moe(ff, experts, top, shared), "mixer": m}


def joint(vocab, width, *layers, eps=1e-5, embed=2.0, side=16):
    return {"architecture": "Garesun", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"scale": embed}, "token_side": {"dim": side}, "layers": list(layers)}


def parallel(vocab, width, *layers, eps=1e-5, taps=3, cap=12.0):
    return {"architecture": "Mebalorn", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "canon": {"taps": taps}, "logit_softcap": cap, "layers": list(layers)}


def config(vocab, width, *layers, eps=1e-5):
    return {"architecture": "Ralesun", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "layers": list(layers)}


CONFIGS = {
    # grouped key heads, both kinds with and without a feed-forward, two windows
    "mixed": config(320, 192, delta(4, 2, 16, 24, 3, ff=320), latent(3, 24, 8, 40, 64, 37),
                    delta(2, 2, 40, 32, 4), latent(5, 16, 16, 32, 48, 70, 500.0, 0.3, ff=256)),
    # two head tiles in decode, window a multiple of nothing, three heads to a key head
    "wide": config(256, 512, latent(20, 64, 32, 64, 160, 100, ff=96), delta(6, 2, 72, 136, 2)),
    # sizes no vector path takes
    "odd": config(203, 100, latent(2, 12, 6, 20, 52, 33, ff=50), delta(3, 1, 20, 17, 5, ff=30)),
    # large latents and heads, more heads than a decode workgroup, long rows of state
    "large": config(128, 256, latent(70, 64, 64, 128, 448, 90), delta(2, 1, 160, 300, 1),
                    latent(17, 128, 64, 136, 512, 64), delta(2, 2, 128, 128, 4)),
    # projections wide enough for the prefill GEMM tiles
    "tiles": config(256, 256, latent(16, 64, 64, 64, 192, 300, ff=512), delta(12, 12, 64, 64, 4, ff=256)),
    # windows of one and two tokens, a window larger than any prompt
    "narrow": config(96, 64, latent(2, 16, 8, 16, 32, 1), latent(2, 16, 8, 16, 32, 2),
                     delta(1, 1, 8, 8, 2), latent(2, 32, 32, 64, 40, 5000, ff=64)),
    # --- the parallel structure: both kinds with and without a feed-forward, grouped heads
    "talking": parallel(320, 192, mingru(88, ff=320), attention(6, 3, 24, 40), mingru(136),
                        attention(4, 1, 40, 24, 0.3, ff=256), cap=5.0),
    # the largest head tiles of the prompt kernels, four heads to a wave, uneven groups
    "talking-wide": parallel(256, 512, attention(20, 5, 64, 96, ff=96), mingru(520, ff=72),
                             attention(32, 8, 128, 128), attention(18, 6, 32, 72), taps=4, cap=25.0),
    # sizes no vector path takes; more taps than usual
    "talking-odd": parallel(203, 99, attention(3, 3, 12, 20, ff=50), mingru(37, ff=30),
                            attention(4, 2, 36, 17), taps=6, cap=9.0),
    # many heads, large heads (no MFMA form), one key head for many; no convolution history
    "talking-any": parallel(128, 256, attention(40, 8, 16, 24, ff=64), attention(2, 1, 136, 200),
                            attention(16, 1, 32, 32), attention(1, 1, 8, 8), taps=1, cap=40.0),
    # projections wide enough for the prefill GEMM tiles, one head to a group, a short convolution
    "talking-tiles": parallel(256, 256, attention(16, 16, 64, 64, ff=512), mingru(512, ff=256),
                              attention(10, 5, 128, 80, ff=256), taps=2),
    # --- norms in groups, convolved projections, capped scores: grouped heads, dense layers, experts
    # in groups and without, a layer that is its mixer alone, values mixed past a layer that does not
    "capped": scaled(320, 192, grouped(6, 2, 24, 40, 16, ff=104, scaling=(4.0, 64, 8.0, 1.0)),
                     grouped(4, 4, 40, 20, 40, conv=4, v_mix=False, cap=9.0),
                     grouped(4, 1, 32, 80, 8, ff=40, experts=8, top=3, groups=(2, 1), base=500.0),
                     grouped(2, 2, 16, 40, 6, conv=2, ff=64, experts=5, top=3, cap=15.0), groups=3),
    # values are mixed from the second layer on; caps too large to do without a running maximum, and
    # none; one expert per token; many heads to a key head
    "capped-wide": scaled(256, 384, grouped(3, 3, 64, 72, 32, v_mix=False, cap=90.0, scale=0.06, ff=200),
                          grouped(20, 1, 128, 96, 64, cap=0.0, scale=0.04, scaling=(8.0, 128, 32.0, 1.0)),
                          grouped(12, 1, 96, 96, 32, conv=4, ff=128, experts=12, top=1, groups=(6, 1)),
                          grouped(8, 4, 72, 24, 24, ff=72, limit=0.7), groups=1, logits=0.7),
    # sizes no vector path takes; more taps than any kernel unrolls
    "capped-odd": scaled(203, 100, grouped(3, 3, 12, 20, 6, conv=7, ff=50),
                         grouped(2, 1, 20, 60, 10, conv=5, ff=30, experts=6, top=4, groups=(2, 2)),
                         grouped(4, 4, 6, 15, 2, conv=1, ff=17, experts=3, top=3), groups=5, mult=1.0),
    # heads no MFMA form takes, a norm group of one lane, taps of one, all experts of a token's group
    "capped-any": scaled(128, 256, grouped(2, 1, 264, 40, 64, conv=1, ff=64, experts=4, top=2, groups=(2, 1)),
                         grouped(1, 1, 200, 40, 0, cap=12.0), grouped(4, 2, 16, 20, 16, ff=96), groups=32),
    # projections and experts wide enough for the prefill GEMM tiles
    "capped-tiles": scaled(256, 256, grouped(16, 4, 128, 128, 64, conv=4, ff=512),
                           grouped(16, 8, 64, 64, 64, ff=256, experts=4, top=2, limit=1.0),
                           grouped(16, 4, 128, 128, 128, conv=4, ff=128, experts=16, top=4, groups=(4, 2), v_mix=False),
                           groups=4),
    # --- one norm for mixer and experts, token inputs: every mixer with and without experts and shared
    # experts, latents read by two layers and a second set of them
    "memory": joint(320, 192, mlstm(2, 32, 48, ff=40, shared=72),
                    gated_latent(5, 24, 8, 40, 48, base=500.0, ff=64, experts=5, top=3),
                    retention(3, 48, 32, 32),
                    gated_latent(3, 16, 8, 24, 48, kv_from=1, base=500.0, scale=0.25, ff=24, experts=4, top=2, shared=40),
                    gated_latent(4, 32, 8, 32, 48, base=500.0),
                    retention(2, 64, 72, 64, base=300.0, ff=32, experts=4, top=4),
                    gated_latent(2, 24, 8, 56, 48, kv_from=4, base=500.0),
                    gated_latent(6, 8, 8, 16, 48, kv_from=1, base=500.0, ff=48, experts=4, shared=16),
                    mlstm(3, 16, 40, cap=4.0), side=24),
    # the largest heads of the chunk kernel, columns over several workgroups, a rotation of a part
    "memory-wide": joint(256, 512, mlstm(4, 128, 128, ff=128, experts=4), retention(2, 256, 200, 128, ff=72, experts=3, shared=64),
                         gated_latent(20, 64, 32, 64, 160), mlstm(1, 144, 320, cap=15.0),
                         gated_latent(17, 128, 32, 96, 160, kv_from=2, ff=64, experts=12, top=11),
                         retention(1, 96, 400, 96), mlstm(2, 256, 256, cap=30.0), embed=1.0, side=64),
    # sizes no vector path takes
    "memory-odd": joint(203, 100, mlstm(3, 20, 17, ff=17, experts=3, top=3), retention(2, 12, 15, 6, ff=9, shared=11),
                        gated_latent(2, 12, 6, 20, 52), gated_latent(3, 10, 6, 9, 52, kv_from=2, ff=21, experts=5),
                        retention(3, 7, 30, 0, decay=[1.0, 0.2, 0.97]), mlstm(1, 130, 261, cap=5.0), side=19),
    # projections and experts wide enough for the prefill GEMM tiles
    "memory-tiles": joint(256, 256, mlstm(8, 64, 64, ff=256, experts=4, shared=256), gated_latent(16, 64, 64, 64, 192),
                          retention(8, 128, 128, 128, ff=128, experts=8, top=4, shared=512),
                          gated_latent(8, 128, 64, 128, 192, kv_from=1, ff=256, experts=4), side=32),
    # recurrent layers only, one of everything
    "memories": joint(96, 64, mlstm(1, 16, 24, ff=24, experts=1, top=1), retention(1, 8, 40, 8), side=20),
    # recurrent layers only
    "average": parallel(96, 64, mingru(24, ff=72), mingru(200), taps=4),
    "recurrent": config(96, 64, delta(2, 2, 24, 16, 4, ff=72), delta(4, 1, 16, 32, 3)),
}


def weights(cfg, seed=0):
    """Random tensors (bf16-representable).  Queries are loud, so that single keys stand out of a
    window, and decays span slow and fast channels.  Routers are loud, so that few choices are
    close calls."""
    g = torch.Generator().manual_seed(seed)
    out = {}

    def put(name, *shape, std=None, mean=0.0):
        std = shape[-1] ** -0.5 if std is None else std
        out[name] = (torch.randn(*shape, generator=g) * std + mean).to(torch.bfloat16)

    def norm(name, W):
        put(name, W, std=0.2, mean=1.0)
        if scaled or side:
            return
        put(name + ".b", W, std=0.1)
        if cfg["architecture"] == "Mebalorn":
            return
        out[name + ".alpha"] = (0.3 + 0.5 * torch.rand((), generator=g)).to(torch.bfloat16)

    V, W, scaled = cfg["vocab"], cfg["width"], cfg["architecture"] == "Nurilorn"
    side = (cfg.get("token_side") or {}).get("dim")
    put("embed", V, W, std=0.5 if scaled or side else 1.5)
    if side:
        put("side.embed", V, len(cfg["layers"]) * side, std=1.0)
    for i, l in enumerate(cfg["layers"]):
        m, p = l["mixer"], f"l{i}.mix."
        norm(f"l{i}.norm1", W)
        if l["type"] == "latent_attention":
            H, R = m["heads"], m["kv_rank"]
            put(p + "q", H * (m["dim"] + m["rot_dim"]), W, std=3 * W ** -0.5)
            if "kv_from" not in m:
                put(p + "dkv", R + m["rot_dim"], W, std=2 * W ** -0.5)
                put(p + "dkv.norm", R, std=0.2, mean=1.0)
            put(p + "uk", H * m["dim"], R)
            put(p + "uv", H * m["vdim"], R)
            if side:
                put(p + "g", H, W, std=1.5 * W ** -0.5)
            else:
                put(p + "sink", H, std=1.0, mean=1.5)
            put(p + "o", W, H * m["vdim"], std=2 * (H * m["vdim"]) ** -0.5)
        elif l["type"] in ("retention", "mlstm"):
            H, d, dv = m["heads"], m["dim"], m["vdim"]
            for x, n in (("q", H * d), ("k", H * d), ("v", H * dv), ("g", H * dv)):
                put(p + x, n, W, std=1.5 * W ** -0.5)
            # a token finds its own key: where one read nothing but it, a chance product near zero
            # would leave the read-out's sign to rounding
            out[p + "k"] = (0.7 * out[p + "k"].float() + 0.7 * out[p + "q"].float()).to(torch.bfloat16)
            if l["type"] == "mlstm":
                for x, mean in (("i", 1.0), ("f", 4.0)):
                    put(p + x, H, W, std=2 * W ** -0.5)
                    put(f"{p}{x}.b", H, std=1.5, mean=mean)
                put(p + "norm", H * dv, std=0.2, mean=1.0)
            put(p + "o", W, H * dv, std=2 * (H * dv) ** -0.5)
        elif scaled:
            H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            for x, n in (("q", H * d), ("k", G * d), ("v", G * dv)):
                put(p + x, n, W, std=(1.0 if x == "v" else 1.7) * W ** -0.5)
                if m["conv"]:
                    put(f"{p}{x}.conv", n, m["conv"], std=0.6)
                    out[f"{p}{x}.conv"][:, -1] += 0.6
            if m["v_mix"]:
                out[p + "vmix"] = (0.3 + 0.3 * torch.rand((), generator=g)).to(torch.bfloat16)
            put(p + "g", H, W, std=1.5 * W ** -0.5)
            put(p + "o", W, H * dv, std=3 * (H * dv) ** -0.5)
            for k in (1, 2) if l["mlp"] else (1,):
                put(f"l{i}.ls{k}", W, std=0.3, mean=0.9)
        elif l["type"] == "attention":
            H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            for x, n in (("q", H * d), ("k", G * d), ("v", G * dv)):
                put(p + x, n, W)
                put(p + x + ".b", n, std=0.8)
            for x in "qk":
                put(p + x + ".norm", d, std=0.4, mean=1.3)
            put(p + "talk", H, H, std=0.8 * H ** -0.5)
            out[p + "talk"] += torch.eye(H).to(torch.bfloat16) * 0.7
            put(p + "sink", H, std=1.0, mean=2.5)
            put(p + "o", W, H * dv, std=2 * (H * dv) ** -0.5)
        elif l["type"] == "mingru":
            C = m["width"]
            for x in "zxg":
                put(p + x, C, W, std=1.5 * W ** -0.5)
            put(p + "z.b", C, std=2.5, mean=-3.0)
            put(p + "x.b", C, std=0.5)
            put(p + "o", W, C, std=3 * C ** -0.5)
        else:
            H, Hk, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            ra, rg = d // 2 + 3, dv // 2 + 1
            for x, n in (("q", Hk * d), ("k", Hk * d), ("v", H * dv)):
                put(p + x, n, W, std=2 * W ** -0.5)
                put(p + x + ".conv", n, m["conv"], std=m["conv"] ** -0.5)
            put(p + "b", H, W, std=2 * W ** -0.5)
            put(p + "A_log", H, std=0.7)
            put(p + "norm", dv, std=0.2, mean=1.0)
            put(p + "a1", ra, W)
            put(p + "a2", H * d, ra)
            put(p + "dt_bias", H * d, std=1.5, mean=-3.0)
            put(p + "g1", rg, W)
            put(p + "g2", H * dv, rg)
            put(p + "o", W, H * dv, std=2 * (H * dv) ** -0.5)
        if l["mlp"] and l["mlp"]["kind"] == "moe":
            ff, n = l["mlp"]["expert"]["ff"], l["mlp"]["router"]["experts"]
            if not side:
                norm(f"l{i}.norm2", W)
            put(f"l{i}.mlp.router", n, W, std=(9 if side else 6) * W ** -0.5)
            if l["mlp"].get("shared"):
                put(f"l{i}.mlp.shared.up", l["mlp"]["shared"]["ff"], W)
                put(f"l{i}.mlp.shared.down", W, l["mlp"]["shared"]["ff"])
            for e in range(n):
                for x in ("gate", "up")[bool(side):]:
                    put(f"l{i}.mlp.e{e}.{x}", ff, W, std=1.5 * W ** -0.5)
                put(f"l{i}.mlp.e{e}.down", W, ff, std=(0.6 if side else 1.2) * ff ** -0.5)
        elif l["mlp"]:
            ff = l["mlp"]["ff"]
            norm(f"l{i}.norm2", W)
            if cfg["architecture"] != "Mebalorn":
                put(f"l{i}.mlp.gate", ff, W, std=2 * W ** -0.5)
            put(f"l{i}.mlp.up", ff, W)
            put(f"l{i}.mlp.down", W, ff, std=2 * ff ** -0.5)
        if side:
            put(f"l{i}.side.gate", side, W)
            put(f"l{i}.side.proj", W, side)
            put(f"l{i}.side.norm", W, std=0.2, mean=0.6)
        if cfg["architecture"] == "Mebalorn":
            for k in (1, 2) if l["mlp"] else (1,):
                put(f"l{i}.canon{k}", W, cfg["canon"]["taps"], std=0.5)
    norm("final.norm", W)
    put("head", V, W, std=(2 if scaled or side else 3 if "logit_softcap" in cfg else 1) * W ** -0.5)
    return out


def save_checkpoint(path, cfg, tensors) -> str:
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    names, head, data = sorted(tensors), {}, b""
    kinds = {torch.bfloat16: "BF16", torch.float32: "F32", torch.int32: "I32"}
    for n in names:
        t = tensors[n].contiguous()
        raw = t.reshape(-1).view(torch.uint8).numpy().tobytes()
        head[n] = {"dtype": kinds[t.dtype], "shape": list(t.shape),
                   "data_offsets": [len(data), len(data) + len(raw)]}
        data += raw
    blob = json.dumps(head).encode()
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(blob)) + blob + data)
    return str(path)


def tokens(cfg, n, seed):
    g = torch.Generator().manual_seed(1000 + seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


def row_errors(got, want):
    """RMS of each row's difference (mean taken off) over the RMS of all of ``want``."""
    d = got.double().cpu() - want.double().cpu()
    d = d - d.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / want.double().std()
