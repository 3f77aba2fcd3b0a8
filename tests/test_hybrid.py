"""Models of mixed layer kinds, and the mechanisms of the Ralesun design (those of the others:
test_hybrid_parallel.py, test_hybrid_grouped.py, test_hybrid_joint.py), against the plain implementation in hybrid_oracle.py: every
mechanism alone, then the model on the engine - portions, batches, reuse of pages and slots,
long decoding, generation.  Each case runs on the CPU (fp32 op references) and, marked gpu, on
the HIP kernels in fp32 and bf16."""
import json
import math
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import hybrid_oracle as O
from hybrid_util import (CONFIGS, attention, config, delta, gated_latent, grouped, joint, latent, mingru, mlstm,
                         parallel, retention, row_errors, save_checkpoint, scaled, tokens, weights)

from drtc_amd import ops
from drtc_amd.engine import LLMEngine, Request, SamplingParams
from drtc_amd.models import (GARESUN_5B, GARESUN_24B, MEBALORN_2B, NURILORN_5B, NURILORN_24B, RALESUN_2B,
                             TINY_GARESUN, TINY_MEBALORN, TINY_NURILORN, TINY_RALESUN, HybridLM, build_model, config_from_dict, get_config, load_model)
from drtc_amd.models.checkpoint import read_safetensors

F32, BF16 = torch.float32, torch.bfloat16
TARGETS = [pytest.param(("cpu", F32), id="cpu"),
           pytest.param(("cuda", F32), id="gpu-f32", marks=pytest.mark.gpu),
           pytest.param(("cuda", BF16), id="gpu-bf16", marks=pytest.mark.gpu)]
on = pytest.mark.parametrize("target", TARGETS)


def tol(dtype, f32, bf16):
    return f32 if dtype == F32 else bf16


def close(got, want, rtol):
    d = (got.double().cpu() - want.double().cpu()).abs().max().item()
    assert d <= rtol * max(1.0, want.double().abs().max().item()), d


def rnd(*shape, seed=0, dtype=F32, dev="cpu", std=1.0):
    """Random values exact in ``dtype``, and the same in float64."""
    t = (torch.randn(*shape, generator=torch.Generator().manual_seed(seed)) * std).to(dtype)
    return t.to(dev), t.double()


# ------------------------------------------------------------------ mechanisms
@on
@pytest.mark.parametrize("rows,W", [(3, 256), (17, 100), (1, 8)])
def test_dynamic_tanh(target, rows, W):
    dev, dt = target
    h, h64 = rnd(rows, W, seed=1, dev=dev, std=3)
    y, y64 = rnd(rows, W, seed=2, dtype=dt, dev=dev)
    w, w64 = rnd(W, seed=3, dev=dev)
    b, b64 = rnd(W, seed=4, dev=dev)
    out = ops.dyt(h, w, b, 0.7, y=y, dtype=dt)
    close(h, h64 + y64, 1e-6)  # the residual stream keeps 32 bits
    close(out, O.dynamic_tanh(h64 + y64, w64, b64, 0.7), tol(dt, 2e-6, 5e-3))
    e, e64 = rnd(11, W, seed=5, dtype=dt, dev=dev)
    ids = torch.arange(rows, dtype=torch.int32, device=dev) % 11
    out = ops.dyt(h, w, b, -1.3, ids=ids, embed=e, dtype=dt)
    close(h, e64[ids.long().cpu()], 0)
    close(out, O.dynamic_tanh(e64[ids.long().cpu()], w64, b64, -1.3), tol(dt, 2e-6, 5e-3))


@on
@pytest.mark.parametrize("dims,rot", [(16, 16), (6, 6), (8, 12)])
def test_latent_rows(target, dims, rot):
    """Latent norm, interleaved rotation (also of a part of the rotated dims, and far out),
    cache write, gather."""
    dev, dt = target
    H, dim, R, base, n = 3, 16, 40, 321.0, 7
    dq = dim + rot
    LW = ops.latent_width(R, rot)
    off = -(-H * dq // 8) * 8
    proj, p64 = rnd(n, off + R + rot + 5, seed=1, dtype=dt, dev=dev)
    w, w64 = rnd(R, seed=2, dev=dev)
    pos = torch.tensor([0, 1, 2, 31, 700, 701, 1023], dtype=torch.int32)
    slots = torch.tensor([32, 33, -1, 95, 64, 40, 41])
    cache = torch.full((3, 32, LW), 7.0, dtype=dt, device=dev)
    lat = torch.empty(n, LW, dtype=dt, device=dev)
    qa = torch.full((n, H, LW), 3.0, dtype=dt, device=dev)
    cs = ops.build_interleaved_rope(1024, dims, base, dev)
    args = (off, H, dim, rot, dims, R, w, 1e-5, cs, pos.to(dev), slots.to(dev), cache)
    ops.latent_prep(proj, *args, qa=qa)
    ops.latent_prep(proj, *args, lat=lat)
    kv = p64[:, off:off + R + rot]
    want = torch.zeros(n, LW, dtype=torch.float64)
    want[:, :R] = O.rms(kv[:, :R], 1e-5) * w64
    want[:, R:R + rot] = O.rotate_interleaved(kv[:, R:], pos, base, dims)
    t = tol(dt, 1e-5, 1e-2)
    close(lat, want, t)
    q = O.rotate_interleaved(p64[:, :H * dq].reshape(n, H, dq)[..., dim:], pos, base, dims)
    close(proj[:, :H * dq].reshape(n, H, dq)[..., dim:], q, t)
    close(qa[..., R:R + rot], q, t)
    assert (qa[..., R + rot:] == 0).all() and (qa[..., :R] == 3).all()
    flat = cache.view(-1, LW)
    for i, s in enumerate(slots.tolist()):
        if s >= 0:
            close(flat[s], want[i], t)
    untouched = [i for i in range(96) if i not in slots.tolist()]
    assert (flat[untouched] == 7).all()
    got = ops.latent_gather(cache, torch.tensor([95, -1, 32], device=dev))
    close(got, torch.stack([want[3], want[0] * 0, want[0]]), t)


def _attention_case(dev, dt, H, dim, rot, vdim, window, lens, ctxs, loud=None, sink=True, seed=0):
    """Random packed portions; ``loud`` (portion, query, key): that score is made to stand
    out.  -> (kernel output rows, float64 expectation, rows)."""
    dq, R = dim + rot, 16
    voff = -(-H * dim // 8) * 8
    n, K = sum(lens), sum(lens) + sum(ctxs)
    q = torch.randn(n, H * dq, generator=torch.Generator().manual_seed(seed))
    kv = torch.randn(K, voff + H * vdim, generator=torch.Generator().manual_seed(seed + 1))
    lat = torch.randn(K, ops.latent_width(R, rot), generator=torch.Generator().manual_seed(seed + 2))
    q_cu = np.concatenate([[0], np.cumsum(lens)])
    k_cu = np.concatenate([[0], np.cumsum(np.add(lens, ctxs))])
    if loud:
        s, i, j = loud
        lat[k_cu[s] + j, R:R + rot] *= 3
        q[q_cu[s] + i].view(H, dq)[:, dim:] = 2 * lat[k_cu[s] + j, R:R + rot]
        kv[k_cu[s] + j, voff:] *= 4
    q, kv, lat = (t.to(dt) for t in (q, kv, lat))
    sk = torch.randn(H, generator=torch.Generator().manual_seed(seed + 3)) + 2 if sink else None
    scale = dq ** -0.5
    qt = ops.latent_qtile(max(lens), dim, rot, vdim)
    ts, tq = ops.portion_tiles(q_cu.tolist(), qt)
    i32 = lambda x: torch.as_tensor(np.asarray(x), dtype=torch.int32, device=dev)
    keys = ops.PortionKeys(i32(k_cu), i32(ctxs), None, k_cu.tolist(), list(ctxs))
    out = torch.full((n, H * vdim), float("nan"), dtype=dt, device=dev)
    ops.latent_prefill_attention(q.to(dev), kv.to(dev), voff, lat.to(dev), R, H, dim, rot, vdim,
                                 i32(q_cu), q_cu.tolist(), keys, (i32(ts), i32(tq)), qt, window,
                                 scale, None if sk is None else sk.to(dev), out)
    want = torch.empty(n, H * vdim, dtype=torch.float64)
    for s, (m, c) in enumerate(zip(lens, ctxs)):
        qs = q[q_cu[s]:q_cu[s + 1]].double().view(m, H, dq)
        ks, ls = kv[k_cu[s]:k_cu[s + 1]].double(), lat[k_cu[s]:k_cu[s + 1]].double()
        sc = scale * (torch.einsum("ihd,jhd->hij", qs[..., :dim], ks[:, :H * dim].reshape(-1, H, dim))
                      + torch.einsum("ihr,jr->hij", qs[..., dim:], ls[:, R:R + rot]))
        ok = O.window_mask(m + c, window)[c:]
        p = O.sink_softmax(sc, ok, None if sk is None else sk.double())
        want[q_cu[s]:q_cu[s + 1]] = torch.einsum(
            "hij,jhv->ihv", p, ks[:, voff:].reshape(-1, H, vdim)).reshape(m, -1)
    return out, want


@on
@pytest.mark.parametrize("dims", [(3, 24, 8, 40), (2, 128, 64, 128), (1, 160, 64, 200), (2, 12, 6, 20)],
                         ids=str)
@pytest.mark.parametrize("window", [1, 33, 64, 150, None])
def test_latent_prefill_attention(target, dims, window):
    dev, dt = target
    reach = [ops.window_reach(s, window) for s in (0, 90, 3, 200, 0)]
    for sink in (True, False):
        out, want = _attention_case(dev, dt, *dims, window, [70, 2, 1, 131, 300], reach, sink=sink)
        close(out, want, tol(dt, 2e-5, 2e-2))


@on
@pytest.mark.parametrize("back", [0, 1, 49, 50, 51, 63, 64])
def test_window_edge_in_prompts(target, back):
    """One key ``back`` tokens behind its query outshines all others: seen inside the window
    of 50, gone outside it, wherever the portion was cut."""
    dev, dt = target
    for start, query in ((0, 100), (0, 64), (77, 0), (77, 40), (200, 63)):
        ctx = ops.window_reach(start, 50)
        key = ctx + query - back
        if not 0 <= key:
            continue
        out, want = _attention_case(dev, dt, 2, 32, 16, 64, 50, [128], [ctx], (0, query, key), seed=back)
        close(out, want, tol(dt, 2e-5, 2e-2))
        v = want[query].abs().max()
        assert (v > 4) == (back < 50)  # the loud key shows (or not) in what is expected


@on
@pytest.mark.parametrize("H,R,rot", [(4, 48, 16), (20, 160, 32), (70, 512, 64), (3, 52, 6), (33, 448, 64)])
def test_latent_decode_attention(target, H, R, rot):
    """Paged rows, windows at and beside block borders, a loud key just inside and just
    outside, splits of the window, padding rows."""
    dev, dt = target
    LW, nb = ops.latent_width(R, rot), 12
    ctx = [1, 2, 32, 33, 64, 95, 96, 97, 160, 310, 0]
    B = len(ctx)
    g = torch.Generator().manual_seed(3)
    cache = (torch.randn(B * nb + 1, 32, LW, generator=g) * 0.7).to(dt)
    cache[..., R + rot:] = 0
    bt = torch.randperm(B * nb, generator=g).view(B, nb).to(torch.int32) + 1
    qa = (torch.randn(B, H, LW, generator=g) * 0.5).to(dt)
    qa[..., R + rot:] = 0
    sink = torch.randn(H, generator=g) + 1
    for window, edge in ((50, 49), (50, 50), (64, 63), (64, 64), (1, 0), (None, 0), (97, 96)):
        c2, q2 = cache.clone(), qa.clone()
        for b, n in enumerate(ctx):  # the key at distance ``edge`` from the last token
            j = n - 1 - edge
            if j >= 0:
                row = c2[bt[b, j // 32], j % 32]
                row[:R + rot] = (q2[b, 0, :R + rot].float() * 4).to(dt)
        for parts in (4, 1):
            ws = None
            if dev == "cuda":
                ws = ops.LatentDecodeWorkspace(B, H, R, window, nb, dev)
                ws.per, ws.splits = -(-nb // parts), parts
                ws.part_o = torch.empty(B, H, parts, R, device=dev)
                ws.part_ml = torch.empty(B, H, parts, 2, device=dev)
            out = ops.latent_decode_attention(q2.to(dev), c2.to(dev), R, bt.to(dev),
                                              torch.tensor(ctx, dtype=torch.int32, device=dev),
                                              window, 0.11, sink.to(dev), ws)
            for b, n in enumerate(ctx):
                if n == 0:
                    assert (out[b] == 0).all()
                    continue
                rows = c2[bt[b].long()].reshape(-1, LW)[:n].double()
                ok = O.window_mask(n, window)[-1:]
                sc = (q2[b].double() @ rows.T * 0.11)[:, None]
                p = O.sink_softmax(sc, ok, sink.double())[:, 0]
                close(out[b], p @ rows[:, :R], tol(dt, 2e-5, 2e-2))


@on
@pytest.mark.parametrize("B,H,N,K", [(1, 3, 64, 24), (5, 2, 40, 16), (70, 4, 20, 128), (3, 2, 13, 7)])
def test_head_linear(target, B, H, N, K):
    dev, dt = target
    x, x64 = rnd(B, H, K + 8, seed=1, dtype=dt, dev=dev)
    w, w64 = rnd(H, N, K, seed=2, dtype=dt, dev=dev)
    out = torch.full((B, H, N + 8), 5.0, dtype=dt, device=dev)
    ops.head_linear(x, w, out=out)
    close(out[..., :N], torch.einsum("bhk,hnk->bhn", x64[..., :K], w64), tol(dt, 1e-5, 1e-2))
    assert (out[..., N:] == 5).all()


def _delta_case(dev, dt, H, Hk, d, dv, taps, lens, seed=0):
    """Whole random sequences: packed inputs on ``dev`` and the oracle's outputs."""
    C = 2 * Hk * d + H * dv
    off_b = -(-C // 8) * 8
    n = sum(lens)
    proj, p64 = rnd(n, off_b + -(-H // 8) * 8, seed=seed, dtype=dt, dev=dev)
    decay, a64 = rnd(n, H * d, seed=seed + 1, dtype=dt, dev=dev)
    gate, g64 = rnd(n, H * dv, seed=seed + 2, dtype=dt, dev=dev)
    conv, c64 = rnd(taps, C, seed=seed + 3, dev=dev, std=taps ** -0.5)
    a_log = torch.linspace(-1.5, 1.5, H, dtype=torch.float64)
    dtb, b64 = rnd(H * d, seed=seed + 5, dev=dev, std=2)
    nw, n64 = rnd(dv, seed=seed + 6, dev=dev)
    w = ops.DeltaWeights(conv, a_log.exp().to(F32).to(dev), dtb, nw, 1e-5, H, Hk, d, dv)
    outs, states = [], []
    r = 0
    for m in lens:
        s = slice(r, r + m)
        r += m
        x = O.silu(O.causal_conv(p64[s, :C], c64.T))
        q = O.unit(x[:, :Hk * d].reshape(m, Hk, d)) * d ** -0.5
        k = O.unit(x[:, Hk * d:2 * Hk * d].reshape(m, Hk, d))
        of = torch.arange(H) // (H // Hk)
        raw = a64[s] + b64
        g = torch.exp(-a_log.exp()[None, :, None] * torch.logaddexp(raw, raw * 0).reshape(m, H, d))
        o, S = O.delta_scan(q[:, of], k[:, of], x[:, 2 * Hk * d:].reshape(m, H, dv), g,
                            torch.sigmoid(p64[s, off_b:off_b + H]))
        o = O.rms(o, 1e-5) * n64 * torch.sigmoid(g64[s]).reshape(m, H, dv)
        outs.append(o.reshape(m, -1))
        states.append(S)
    return proj, off_b, w, decay, gate, torch.cat(outs), states


def _portions(dev, lens, poss, slots):
    i32 = lambda x: torch.as_tensor(np.asarray(x, np.int64), dtype=torch.int32, device=dev)
    row = np.concatenate([[0], np.cumsum(lens)[:-1]])
    off = np.concatenate([np.arange(n) for n in lens])
    p = ops.Portions(i32(row), i32(lens), i32(poss), i32(slots), i32(off), i32(np.repeat(slots, lens)),
                     max(lens))
    return p, i32(off + np.repeat(poss, lens))


DELTA_SHAPES = [(4, 2, 16, 24, 3), (2, 2, 128, 128, 4), (3, 1, 72, 136, 2), (2, 1, 160, 300, 1),
                (3, 3, 20, 17, 5), (1, 1, 64, 80, 4)]


@on
@pytest.mark.parametrize("shape", DELTA_SHAPES, ids=str)
@pytest.mark.parametrize("columns", [0, 2, 4])
def test_delta_rule(target, shape, columns):
    """Packed whole sequences, then the same cut into portions and single decoded tokens, in
    state slots that hold another sequence's leftovers."""
    dev, dt = target
    H, Hk, d, dv, taps = shape
    lens = [37, 1, 2, 18]
    proj, off_b, w, decay, gate, want, states = _delta_case(dev, dt, *shape, lens)
    t = tol(dt, 5e-5, 3e-2)

    def fresh():
        return (torch.full((5, taps, w.channels), 9.0, dtype=dt, device=dev),
                torch.full((5, H, d, dv), 9.0, device=dev))

    ring, state = fresh()
    slots = [3, 0, 4, 1]
    p, pos = _portions(dev, lens, [0] * 4, slots)
    conv = ops.short_conv(proj, w, ring, pos, p)
    out = ops.delta_scan(proj, off_b, conv, w, ring, state, decay, gate, p, columns)
    close(out, want, t)
    for s, S in zip(slots, states):
        close(state[s], S, t)
    assert (state[2] == 9).all() and (ring[2] == 9).all()

    # sequence 0 in portions and single tokens
    ring, state = fresh()
    rows, a = [], 0
    for n in (2, 5, 1, 16, 2, 1, 1, 9):
        s = slice(a, a + n)
        if n == 1:
            pos = torch.tensor([a, 0], dtype=torch.int32, device=dev)  # and a padding row
            two = slice(a, a + 2)
            o = ops.delta_decode(proj[two].contiguous(), off_b, w, ring, state, decay[two], gate[two],
                                 pos, torch.tensor([2, -1], dtype=torch.int32, device=dev))
            assert (o[1] == 0).all()
            rows.append(o[:1])
        else:
            p, pos = _portions(dev, [n], [a], [2])
            x = proj[s].contiguous()
            conv = ops.short_conv(x, w, ring, pos, p)
            rows.append(ops.delta_scan(x, off_b, conv, w, ring, state, decay[s], gate[s], p, columns))
        a += n
    assert a == 37
    close(torch.cat(rows), want[:37], t)
    close(state[2], states[0], t)


@on
def test_delta_remembers_far_tokens(target):
    """Channels that hardly decay: a loud write hundreds of tokens back still shows."""
    dev, dt = target
    proj, off_b, w, decay, gate, _, _ = _delta_case(dev, dt, 1, 1, 32, 32, 2, [400])
    decay.fill_(-12.0)
    w.dt_bias.zero_()
    outs = []
    for loud in (False, True):
        x = proj.clone()
        if loud:
            x[3, 64:96] *= 30
        ring = torch.zeros(1, 2, w.channels, dtype=dt, device=dev)
        state = torch.zeros(1, 1, 32, 32, device=dev)
        x[:, off_b] = -8.0  # hardly any later writes
        x[3, off_b] = 8.0
        p, pos = _portions(dev, [400], [0], [0])
        conv = ops.short_conv(x, w, ring, pos, p)
        outs.append(ops.delta_scan(x, off_b, conv, w, ring, state, decay, gate, p))
    assert (outs[0][:3] == outs[1][:3]).all()
    assert (outs[0][399].float() - outs[1][399].float()).abs().max() > 0.05


@on
def test_gated_feed_forward(target):
    dev, dt = target
    x, x64 = rnd(9, 64, seed=1, dtype=dt, dev=dev)
    gu, g64 = rnd(2 * 96, 64, seed=2, dtype=dt, dev=dev, std=0.25)
    dn, d64 = rnd(64, 96, seed=3, dtype=dt, dev=dev, std=0.2)
    y = ops.linear(ops.gated(x, gu, "gelu_tanh"), dn)
    close(y, O.gated_mlp(x64, {"gate": g64[:96], "up": g64[96:], "down": d64}), tol(dt, 1e-5, 2e-2))


# ------------------------------------------------------------------ the model
_cache: dict = {}


def case(name, seed=0):
    """(config dict, weights) of a test model."""
    key = (name, seed)
    if key not in _cache:
        _cache[key] = (CONFIGS[name], weights(CONFIGS[name], seed))
    return _cache[key]


def oracle(cfg, w, toks):
    """Logits, and in a further column how close the closest routing decision is that the position
    or the few tokens behind it (which its convolutions read) depend on."""
    margins = []
    lg = O.forward(cfg, w, toks, margins)[0]
    near = torch.full((len(toks),), math.inf, dtype=lg.dtype)
    for m in margins:
        for back in range(4):
            near[back:] = torch.minimum(near[back:], m[:max(len(m) - back, 0)])
    return torch.cat([lg, near[:, None]], 1)


def expected(name, toks):
    key = (name, tuple(toks))
    if key not in _cache:
        _cache[key] = oracle(*case(name), toks)
    return _cache[key]


def engine(name, target, max_batch=4, max_len=512, blocks=None, **kw):
    dev, dt = target
    cfg, w = case(name)
    m = build_model(config_from_dict(cfg).replace(max_position=max_len), dev, dtype=dt, tensors=w)
    return LLMEngine(m, max_batch=max_batch, max_model_len=max_len,
                     num_blocks=blocks or max_batch * (-(-max_len // 32)) + 1, **kw)


def feed_all(eng, toks, cuts):
    """Logits of every position, the sequence cut into portions of ``cuts`` (the last repeats)."""
    r, out, a, i = Request([]), [], 0, 0
    while a < len(toks):
        n = min(cuts[min(i, len(cuts) - 1)], len(toks) - a)
        out += eng.feed([(r, toks[a:a + n], list(range(n)))])
        a += n
        i += 1
    eng.release(r)
    return torch.cat(out)


def agree(got, want, dtype):
    few = 0
    if want.shape[1] > got.shape[1]:
        # a choice of experts that bf16 may see otherwise changes the token for good, and a little
        # what later tokens see of it
        sure = want[:, -1] > (0.15 if dtype == BF16 else 1e-4)
        assert not torch.isnan(got).any() and sure.sum() >= 0.3 * len(sure) - 1
        if not sure.any():
            return
        few = max(1, len(want) // 30) if dtype == BF16 and not sure.all() else 0
        got, want = got[sure.to(got.device)], want[sure, :-1]
    e = row_errors(got, want)
    assert not torch.isnan(e).any()
    # a few positions amplify bf16 rounding (a short read-out, divided by its own size)
    limit = tol(dtype, 2e-4, 0.2)
    assert (e > limit).sum() <= few, (int(e.argmax()), float(e.max()))
    assert (e > 0.1).sum() <= max(1, e.numel() // 50) + few


@on
@pytest.mark.parametrize("name", list(CONFIGS))
def test_prompt_decode_and_portions(target, name):
    """Whole prompt, token by token, and portions down to two tokens agree with the oracle at
    every position: first tokens, window edges, block borders."""
    cfg, _ = case(name)
    n = 150
    toks = tokens(cfg, n, 1)
    want = expected(name, toks)
    eng = engine(name, target)
    cuts = [[n], [1], [31, 2, 3, 2, 29, 1, 1, 16], [2]]
    if target[0] == "cpu":
        cuts = cuts[:3]
    for c in cuts:
        agree(feed_all(eng, toks, c), want, target[1])
    assert eng.alloc.num_used == 0 and eng.kv.states.num_used == 0


@on
@pytest.mark.parametrize("name", ["mixed", "talking", "capped", "memory"])
def test_stream_follows_the_oracle(target, name):
    """The residual stream after every layer (fp32)."""
    dev, dt = target
    cfg, w = case(name)
    toks = tokens(cfg, 90, 2)
    m = build_model(config_from_dict(cfg), dev, dtype=dt, tensors=w)
    agree(m.forward_reference([toks])[0], oracle(cfg, w, toks), dt)
    # a model that ends after layer i shows that layer's stream through an identity-like head
    for i in range(len(cfg["layers"])):
        c2 = dict(cfg, layers=cfg["layers"][:i + 1], vocab=cfg["width"])
        w2 = {k: v for k, v in w.items() if not k.startswith("l") or int(k[1:k.index(".")]) <= i}
        if "side.embed" in w:
            w2["side.embed"] = w["side.embed"][:cfg["width"], :(i + 1) * cfg["token_side"]["dim"]]
        w2["embed"] = w["embed"][:cfg["width"]]
        w2["head"] = torch.eye(cfg["width"]).to(BF16)
        t2 = [t % cfg["width"] for t in toks]
        m2 = build_model(config_from_dict(c2), dev, dtype=dt, tensors=w2)
        agree(m2.forward_reference([t2])[0], oracle(c2, w2, t2), dt)


@on
@pytest.mark.parametrize("name", ["mixed", "wide", "odd", "talking", "talking-wide", "talking-odd", "talking-any",
                                  "capped", "capped-wide", "capped-odd", "capped-any", "memory", "memory-wide",
                                  "memory-odd"])
def test_mixed_batches(target, name):
    """Portions beside single tokens of other requests, idle requests, unequal lengths, and
    pages and slots freed and taken again - from a pool that holds no more than the live
    requests."""
    cfg, _ = case(name)
    lens = [130, 9, 64, 33, 70, 2, 97, 40]
    seqs = [tokens(cfg, n, 10 + i) for i, n in enumerate(lens)]
    rng = np.random.default_rng(5)
    eng = engine(name, target, max_len=160, blocks=14)
    live, todo, at, got = {}, list(range(len(seqs))), {}, {i: [] for i in range(len(seqs))}
    kinds = set()
    while todo or live:
        while todo and len(live) < 4 and \
                sum(-(-lens[i] // 32) for i in [*live, todo[0]]) <= 13:
            live[todo[0]] = Request([])
            at[todo.pop(0)] = 0
        entries, who = [], []
        for i, r in live.items():
            if len(live) > 1 and rng.random() < 0.2:
                continue  # left out of this step
            n = 1 if rng.random() < 0.4 else int(rng.choice([2, 3, 17, 40]))
            n = min(n, lens[i] - at[i])
            entries.append((r, seqs[i][at[i]:at[i] + n], list(range(n))))
            who.append(i)
        if not entries:
            continue
        kinds.add((any(len(e[1]) > 1 for e in entries), any(len(e[1]) == 1 for e in entries)))
        for i, (r, t, _), o in zip(who, entries, eng.feed(entries)):
            got[i].append(o)
            at[i] += len(t)
            if at[i] == lens[i]:
                eng.release(live.pop(i))
    assert kinds == {(True, True), (True, False), (False, True)}
    for i, s in enumerate(seqs):
        agree(torch.cat(got[i]), expected(name, s), target[1])
    assert eng.alloc.num_used == 0 and eng.kv.states.num_used == 0


@on
@pytest.mark.parametrize("name", ["mixed", "talking", "capped", "memory"])
def test_unwanted_rows_still_count(target, name):
    """Steps nothing is asked of leave the same cache and state; wanted places come in order."""
    cfg, _ = case(name)
    toks = tokens(cfg, 60, 4)
    want = expected(name, toks)
    eng = engine(name, target)
    r, s = Request([]), Request([])
    assert eng.feed([(r, toks[:20], [])])[0].shape == (0, cfg["vocab"])
    a, b = eng.feed([(r, toks[20:21], []), (s, toks[:50], [40, 3, 3])])
    assert a.shape[0] == 0
    agree(b, want[[40, 3, 3]], target[1])
    eng.feed([(r, toks[21:22], [])])
    b, a = eng.feed([(s, toks[50:], [9]), (r, toks[22:], [0, 37])])
    agree(a, want[[22, 59]], target[1])
    agree(b, want[[59]], target[1])


@on
@pytest.mark.parametrize("name", ["mixed", "talking", "capped", "memory"])
def test_long_decoding(target, name):
    """Hundreds of decoded tokens: windows, splits and blocks pass over decoded tokens."""
    if target[0] == "cpu":
        n, start = 230, 100
    else:
        n, start = 480, 5
    cfg, _ = case(name)
    toks = tokens(cfg, n, 6)
    agree(feed_all(engine(name, target), toks, [start, 1]), expected(name, toks), target[1])


@pytest.mark.gpu
@pytest.mark.parametrize("name", ["tiles", "talking-tiles", "talking-wide", "capped-tiles", "capped-wide", "memory-tiles",
                                  "memory-wide"])
@pytest.mark.parametrize("dtype", [F32, BF16], ids=["f32", "bf16"])
def test_prefill_sized_steps(dtype, name):
    """Steps of more than a thousand rows (the prefill GEMMs, 256-row query tiles, portions far
    into a prompt) beside decode rows."""
    cfg, _ = case(name)
    a, b, c = (tokens(cfg, n, n) for n in (1500, 1210, 40))
    ea, eb, ec = (expected(name, t) for t in (a, b, c))
    eng = engine(name, ("cuda", dtype), max_len=1536)
    ra, rb, rc = Request([]), Request([]), Request([])
    got = eng.feed([(ra, a[:700], list(range(700))), (rb, b[:520], list(range(520))), (rc, c[:39], [38])])
    agree(got[0], ea[:700], dtype)
    agree(got[1], eb[:520], dtype)
    got = eng.feed([(rc, c[39:], [0]), (rb, b[520:1200], list(range(680))), (ra, a[700:1400], list(range(700)))])
    agree(got[0], ec[39:], dtype)
    agree(got[1], eb[520:1200], dtype)
    agree(got[2], ea[700:1400], dtype)
    got = [eng.feed([(ra, [a[1400 + i]], [0]), (rb, [b[1200 + i]], [0])]) for i in range(10)]
    agree(torch.cat([g[0] for g in got]), ea[1400:1410], dtype)
    agree(torch.cat([g[1] for g in got]), eb[1200:], dtype)


def _mutations():
    def layers(f):
        return lambda c, w: ({**c, "layers": [f(json.loads(json.dumps(l))) for l in c["layers"]]}, w)

    def window(k):
        def f(l):
            if "mask" in l["mixer"]:
                l["mixer"]["mask"]["size"] += k
            return l
        return layers(f)

    def swap(key, f):
        return lambda c, w: (c, {k: (f(t) if k.endswith(key) else t) for k, t in w.items()})

    def canon(f):
        return lambda c, w: (c, {k: (f(t) if ".canon" in k else t) for k, t in w.items()})

    def one_norm(c, w):
        return c, {k: (w[k.replace("norm2", "norm1")] if "norm2" in k else t) for k, t in w.items()}

    def mixer(f):
        def g(l):
            f(l["mixer"])
            return l
        return layers(g)

    def every_value(c, w):  # a layer that should leave its values alone
        w = dict(w)
        w["l1.mix.vmix"] = torch.tensor(0.5)
        return mixer(lambda m: m.update(v_mix=True))(c, w)

    def no_groups(l):
        if l["mlp"] and l["mlp"]["kind"] == "moe":
            l["mlp"]["router"].pop("groups", None)
        return l

    def no_limit(l):
        if l["mlp"]:
            l["mlp"].get("expert", l["mlp"])["limit"] = 1e6
        return l

    def own_read(l):  # the other set of latents
        if l["mixer"].get("kv_from") == 1:
            l["mixer"]["kv_from"] = 4
        return l

    def no_shared(l):
        (l["mlp"] or {}).pop("shared", None)
        return l

    return {("mixed", "window+1"): window(1), ("mixed", "window-1"): window(-1),
            ("mixed", "no sink"): swap(".sink", lambda t: t * 0 - 50),
            ("mixed", "no decay bias"): swap("dt_bias", lambda t: t * 0),
            ("mixed", "taps reversed"): swap(".conv", lambda t: t.flip(-1)),
            ("mixed", "no norm bias"): swap("norm1.b", lambda t: t * 0),
            ("talking", "no sink"): swap(".sink", lambda t: t * 0 - 50),
            ("talking", "talk transposed"): swap(".talk", lambda t: t.t()),
            ("talking", "no talk"): swap(".talk", lambda t: torch.eye(t.shape[0]).to(t.dtype)),
            ("talking", "no query bias"): swap(".q.b", lambda t: t * 0),
            ("talking", "one-plus norm"): swap(".k.norm", lambda t: t + 1),
            ("talking", "taps reversed"): canon(lambda t: t.flip(-1)),
            ("talking", "taps late"): canon(lambda t: torch.roll(t, 1, -1)),
            ("talking", "one norm for both"): one_norm,
            ("talking", "no norm bias"): swap("norm1.b", lambda t: t * 0),
            ("talking", "no gate bias"): swap(".z.b", lambda t: t * 0),
            ("talking", "no cap"): lambda c, w: ({**c, "logit_softcap": 1e6}, w),
            ("capped", "taps reversed"): swap(".conv", lambda t: t.flip(-1)),
            ("capped", "taps late"): swap(".conv", lambda t: torch.roll(t, 1, -1)),
            ("capped", "no value mixing"): swap(".vmix", lambda t: t * 0),
            ("capped", "gates open"): swap(".mix.g", lambda t: t * 0),
            ("capped", "no cap"): mixer(lambda m: m.update(softcap=1e6)),
            ("capped", "rotation unscaled"): mixer(lambda m: m["rot"].pop("scaling", None)),
            ("capped", "mixes every layer"): every_value,
            ("capped", "one norm group"): lambda c, w: ({**c, "norm": {**c["norm"], "groups": 1}}, w),
            ("capped", "no layer scale"): swap(".ls2", lambda t: t * 0 + 1),
            ("capped", "residual not multiplied"): lambda c, w: ({**c, "residual_mult": 1.0}, w),
            ("capped", "experts of any group"): layers(no_groups),
            ("capped", "no limit"): layers(no_limit),
            ("memory", "other latents"): lambda c, w: (dict(c, layers=[
                own_read(json.loads(json.dumps(l))) if i == 7 else l for i, l in enumerate(c["layers"])]), w),
            ("memory", "no shared experts"): layers(no_shared),
            ("memory", "gates open"): swap(".mix.g", lambda t: t * 0),
            ("memory", "input gates shut"): swap(".mix.i.b", lambda t: t - 3),
            ("memory", "no input gate"): swap(".mix.i", lambda t: t * 0),
            ("memory", "no forget bias"): swap(".mix.f.b", lambda t: t * 0),
            ("memory", "forgets later"): swap(".mix.f.b", lambda t: t + 3),
            ("memory", "loose cap"): mixer(lambda m: m.update(gate_cap=1e6) if "gate_cap" in m else None),
            ("memory", "other decay"): mixer(lambda m: m.update(decay=m["decay"][::-1]) if "decay" in m else None),
            ("memory", "no memory norm"): swap(".mix.norm", lambda t: t * 0 + 1),
            ("memory", "rotation"): mixer(lambda m: m["rot"].update(base=50.0) if "decay" in m else None),
            ("memory", "part unrotated"): mixer(lambda m: m["rot"].update(dims=32) if m["dim"] == 64 else None),
            ("memory", "no latent norm"): swap(".dkv.norm", lambda t: t * 0 + 1),
            ("memory", "no token inputs"): swap(".side.norm", lambda t: t * 0),
            ("memory", "another layer's input"): swap("side.embed", lambda t: torch.roll(t, 24, 1)),
            ("memory", "embedding unscaled"): lambda c, w: ({**c, "embedding": {"scale": 1.0}}, w)}


@pytest.mark.parametrize("mistake", list(_mutations()), ids=": ".join)
def test_mistakes_show(mistake):
    """The tests' models and tolerances can tell: each mistake, planted in the oracle, moves
    some logits by more than the loosest limit, several by more than half of it."""
    cfg, w = case(mistake[0])
    toks = tokens(cfg, 150, 1)
    got = O.forward(*_mutations()[mistake](cfg, w), toks)[0]
    e = row_errors(got, expected(mistake[0], toks)[:, :-1])
    assert e.max() > 0.2 and (e > 0.1).sum() > 3


# ------------------------------------------------------------------ scheduler, sampler, command line
def greedy_ok(name, prompt, out, slack):
    """Every generated token maximises the oracle's logits (within ``slack`` and the sampler's bf16)."""
    lg = oracle(*case(name), prompt + out[:-1])[len(prompt) - 1:]
    near, lg = lg[:, -1], lg[:, :-1]
    for j, t in enumerate(out):
        assert near[j] < 0.15 or lg[j, t] >= lg[j].max() - slack - lg[j].abs().max() / 256, j


@on
@pytest.mark.parametrize("name", ["mixed", "talking", "capped", "memory"])
@pytest.mark.parametrize("how", ["whole", "portions", "preempted"])
def test_greedy_generation(target, how, name):
    cfg, _ = case(name)
    prompts = [tokens(cfg, n, 20 + n) for n in (1, 5, 40, 90, 33, 64)]
    new = [6 + 4 * i for i in range(len(prompts))]
    kw = {}
    if how == "preempted":  # four prompts fit, their outputs do not
        prompts, new, kw = [tokens(cfg, n, n) for n in (30, 27, 29, 31)], [45] * 4, {"blocks": 7}
    eng = engine(name, target, max_len=256, **kw)
    if how == "portions":
        eng.prefill_chunk_tokens = 32
        eng.max_prefill_tokens = 48
    reqs = eng.generate(prompts, [SamplingParams.greedy(n, ignore_eos=True) for n in new])
    for p, r, n in zip(prompts, reqs, new):
        assert len(r.output_ids) == n and r.finish_reason == "length"
        greedy_ok(name, p, r.output_ids, tol(target[1], 2e-2, 0.5))
    if how == "preempted":
        assert eng.stats["preemptions"] > 0
    else:
        assert eng.stats["mixed_steps"] > 0
    assert eng.alloc.num_used == 0 and eng.kv.states.num_used == 0


@on
@pytest.mark.parametrize("name", ["mixed", "talking", "capped", "memory"])
def test_generation_with_stops_and_aborts(target, name):
    """Pipelined decoding over a changing batch: stop tokens found a step late, aborts, slot
    moves; every output as alone."""
    cfg, _ = case(name)
    prompts = [tokens(cfg, n, 40 + n) for n in (7, 20, 3, 50, 11)]
    alone = [engine(name, target, max_len=128).generate([p], SamplingParams.greedy(20, ignore_eos=True))[0]
             .output_ids for p in prompts]
    eng = engine(name, target, max_len=128, max_batch=3)
    reqs = []
    for p, a in zip(prompts, alone):
        reqs.append(eng.add_request(Request(list(p), SamplingParams(
            max_new_tokens=20, temperature=0.0, top_k=0, top_p=1.0, stop_token_ids=(a[9],)))))
    gone = eng.add_request(Request(tokens(cfg, 30, 99), SamplingParams.greedy(50)))
    while eng.has_work():
        eng.step()
        if reqs[0].state.value == "finished" and gone.state.value != "finished":
            eng.abort(gone)
    for r, a, p in zip(reqs, alone, prompts):
        if target[1] == F32:
            cut = a.index(a[9]) + 1
            assert r.output_ids == a[:cut], p
        else:
            greedy_ok(name, p, r.output_ids, 0.5)
    assert eng.alloc.num_used == 0 and eng.kv.states.num_used == 0


@pytest.mark.gpu
@pytest.mark.parametrize("name", ["mixed", "talking", "capped", "memory"])
def test_graphs_match_eager(name):
    """Replays of a captured step - several, with eager work between - advance the recurrent
    state exactly once each."""
    for dt in (F32, BF16):
        cfg, _ = case(name)
        prompts = [tokens(cfg, n, 60 + n) for n in (4, 30, 65)]
        outs = []
        for graphs in (True, False):
            eng = engine(name, ("cuda", dt), max_len=256, use_graphs=graphs)
            if graphs:
                eng.warmup()
            a = [r.output_ids for r in eng.generate(prompts, SamplingParams.greedy(15, ignore_eos=True))]
            b = [r.output_ids for r in eng.generate(prompts[1:], SamplingParams.greedy(9, ignore_eos=True))]
            outs.append((a, b))
        assert outs[0] == outs[1]


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
@pytest.mark.parametrize("name", ["mixed", "talking", "capped", "memory"])
def test_trace_run(tmp_path, dtype, name):
    """The command-line replay: files, order, reuse of the pool, exit status."""
    cfg, w = case(name)
    path = save_checkpoint(tmp_path / "model", cfg, w)
    a, b = tokens(cfg, 70, 7), tokens(cfg, 45, 8)
    steps = [{"entries": [{"id": "a", "tokens": a[:40], "want": [39, 2]}, {"id": "b", "tokens": b[:1], "want": [0]}]},
             {"entries": [{"id": "b", "tokens": b[1:44], "want": []}, {"id": "a", "tokens": a[40:41], "want": []}]},
             {"entries": [{"id": "b", "tokens": b[44:], "want": [0]}, {"id": "a", "tokens": a[41:42], "want": [0]}],
              "end": ["b"]},
             {"entries": [{"id": "c", "tokens": b, "want": [44]}, {"id": "a", "tokens": a[42:], "want": [27]}],
              "end": ["a", "c"]}]
    text = "".join(json.dumps({"step": i, "end": [], **s}) + "\n" for i, s in enumerate(steps))
    out = tmp_path / "out"
    out.mkdir()
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    p = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", path, "--dtype", dtype,
                        "--out", str(out), "--max-tokens", "192"], input=text, text=True,
                       capture_output=True, timeout=100)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
    assert sorted(os.listdir(out)) == ["0.f32", "2.f32", "3.f32"]
    ea, eb = expected(name, a), expected(name, b)
    want = {0: [ea[39], ea[2], eb[0]], 2: [eb[44], ea[41]], 3: [eb[44], ea[69]]}
    for i, rows in want.items():
        got = torch.from_numpy(np.fromfile(out / f"{i}.f32", "<f4").reshape(len(rows), -1))
        agree(got, torch.stack(rows), F32 if dtype == "float32" else BF16)


def test_checkpoint_folder(tmp_path):
    cfg, w = case("odd")
    path = save_checkpoint(tmp_path / "m", cfg, w)
    back = read_safetensors(os.path.join(path, "model.safetensors"))
    assert back.keys() == w.keys() and all((back[k] == w[k]).all() and back[k].shape == w[k].shape for k in w)
    c = get_config(path)
    assert c == load_model(path, "cpu").cfg and c.hidden_size == 100 and c.windows == (33,)
    toks = tokens(cfg, 20, 1)
    m = load_model(path, "cpu", dtype=F32, max_position=64)
    agree(m.forward_reference([toks])[0], expected("odd", toks), F32)
    with pytest.raises(KeyError):
        HybridLM(c, "cpu", tensors={k: v for k, v in w.items() if k != "l1.mix.A_log"})
    with pytest.raises(ValueError):
        HybridLM(c, "cpu", tensors={**w, "l1.mix.extra": w["embed"]})
    with pytest.raises(ValueError):
        HybridLM(c, "cpu", tensors={**w, "head": w["head"][:, :-1]})
    with pytest.raises(KeyError):
        config_from_dict(dict(cfg, architecture="other"))
    with pytest.raises(ValueError):
        config_from_dict(dict(cfg, layers=[dict(cfg["layers"][0], type="other")]))
    with open(os.path.join(path, "model.safetensors"), "r+b") as f:
        f.truncate(5000)
    with pytest.raises(ValueError):
        read_safetensors(os.path.join(path, "model.safetensors"))


@on
@pytest.mark.parametrize("cfg", [TINY_RALESUN, TINY_MEBALORN, TINY_NURILORN, TINY_GARESUN], ids=lambda c: c.name)
def test_registered_preset_serves(target, cfg):
    dev, dt = target
    m = build_model(cfg, dev, seed=3, dtype=dt)
    eng = LLMEngine(m, max_batch=4, max_model_len=256)  # cache sized by the manager
    reqs = eng.generate([[1, 5, 9], list(range(1, 80))],
                        SamplingParams(max_new_tokens=10, temperature=0.8, top_k=20, top_p=0.9, ignore_eos=True))
    assert all(len(r.output_ids) == 10 for r in reqs)
    assert m.weight_bytes() > 0 and eng.kv.bytes > 0
    assert m.weight_bytes() >= cfg.num_params() * m.embed.element_size()
    assert abs(RALESUN_2B.num_params() / 2.9e9 - 1) < 0.3
    assert abs(MEBALORN_2B.num_params() / 1.8e9 - 1) < 0.1
    assert abs(GARESUN_5B.num_params() / 5e9 - 1) < 0.2 and abs(GARESUN_24B.num_params() / 24e9 - 1) < 0.2
    assert abs(NURILORN_5B.num_params() / 5e9 - 1) < 0.1 and abs(NURILORN_24B.num_params() / 24e9 - 1) < 0.1


@pytest.mark.parametrize("name", ["mixed", "talking", "capped", "memory"])
def test_service_backend_from_checkpoint_folder(tmp_path, name):
    """The LLM service's --model takes a checkpoint folder; text in, text out."""
    from argparse import Namespace

    from drtc_amd.llm.server import build_backend

    cfg, w = case(name)
    path = save_checkpoint(tmp_path / "m", cfg, w)
    backend = build_backend(Namespace(backend="engine", model=path, max_batch=2, max_model_len=128,
                                      no_graphs=True, tp=1, gpus=1, in_process=True))
    try:
        out = backend.generate(["hello there", "ok"], SamplingParams.greedy(5, ignore_eos=True))
        assert len(out) == 2 and all(isinstance(t, str) for t in out)
    finally:
        backend.close()


def test_limits_are_errors():
    eng = engine("mixed", ("cpu", F32), max_len=64)
    r = Request([])
    with pytest.raises(ValueError):
        eng.feed([(r, [], [])])
    with pytest.raises(ValueError):
        eng.feed([(Request([]), [1] * 65, [])])
    from drtc_amd.parallel.comm import ParallelContext
    with pytest.raises(ValueError):
        build_model(TINY_RALESUN, "cpu", pc=ParallelContext(tp_size=2, tp_rank=0))
    with pytest.raises(ValueError):
        config_from_dict(config(16, 16, delta(3, 2, 8, 8, 2)))
    with pytest.raises(ValueError):
        config_from_dict(config(16, 16, latent(1, 8, 8, 8, 8, 0)))
    for bad in (parallel(16, 16, attention(3, 2, 8, 8)), parallel(16, 16, mingru(0)),
                parallel(16, 16, attention(2, 2, 300, 8)), parallel(16, 16, mingru(8), cap=0.0),
                parallel(16, 16, mingru(8), taps=13), parallel(16, 9000, mingru(8)),
                parallel(16, 16, dict(mingru(8), type="other")),
                scaled(16, 16, grouped(3, 2, 8, 8, 8)), scaled(16, 16, grouped(2, 2, 8, 8, 7)),
                scaled(16, 16, grouped(2, 2, 8, 8, 10)), scaled(16, 15, grouped(2, 2, 8, 8, 8)),
                scaled(16, 16, grouped(2, 2, 8, 8, 8, ff=8, limit=0.0)),
                scaled(16, 16, grouped(2, 2, 8, 8, 8), grouped(2, 1, 8, 8, 8)),
                scaled(16, 16, grouped(2, 2, 8, 8, 8, ff=8, experts=6, top=2, groups=(4, 1))),
                scaled(16, 16, grouped(2, 2, 8, 8, 8, ff=8, experts=6, top=4, groups=(2, 1))),
                scaled(16, 16, dict(grouped(2, 2, 8, 8, 8), type="other")),
                scaled(16, 16, dict(grouped(2, 2, 8, 8, 8), mlp={"kind": "other"})),
                joint(16, 16, retention(2, 8, 8, decay=[0.5])), joint(16, 16, retention(1, 8, 8, decay=[1.5])),
                joint(16, 16, retention(1, 8, 8, decay=[0.0])), joint(16, 16, retention(1, 8, 8, 10)),
                joint(16, 16, retention(1, 300, 8)), joint(16, 16, mlstm(1, 8, 1100)),
                joint(16, 16, mlstm(1, 8, 8, cap=0.0)), joint(16, 16, dict(mlstm(1, 8, 8), type="other")),
                joint(16, 16, dict(mlstm(1, 8, 8), mlp={"kind": "other"})),
                joint(16, 16, mlstm(1, 8, 8, ff=8, experts=4, top=5)),
                joint(16, 16, gated_latent(1, 8, 8, 8, 8, kv_from=0)),
                joint(16, 16, mlstm(1, 8, 8), gated_latent(1, 8, 8, 8, 8, kv_from=0)),
                joint(16, 16, gated_latent(1, 8, 8, 8, 8), gated_latent(1, 8, 8, 8, 16, kv_from=0)),
                joint(16, 16, gated_latent(1, 8, 8, 8, 8), gated_latent(1, 8, 8, 8, 8, base=5.0, kv_from=0)),
                joint(16, 16, gated_latent(1, 8, 8, 8, 8), gated_latent(1, 8, 8, 8, 8, kv_from=0),
                      gated_latent(1, 8, 8, 8, 8, kv_from=1))):
        with pytest.raises(ValueError):
            config_from_dict(bad)
    with pytest.raises(ValueError):
        build_model(TINY_MEBALORN, "cpu", pc=ParallelContext(tp_size=2, tp_rank=0))
    assert math.isclose(config_from_dict(config(16, 16, latent(1, 8, 8, 8, 8, 3))).layers[0].mixer.scale, 0.25)
