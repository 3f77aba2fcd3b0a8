"""The mechanisms of joint layers, each alone against hybrid_oracle.py: retention and matrix memory
(portions, decoded tokens, reused slots, far keys), the layer norm behind a token's side input, head
gates and shared latents of latent attention, squared-relu experts added to the stream.  On the CPU
(fp32 op references) and, marked gpu, on the HIP kernels in fp32 and bf16."""
import numpy as np
import pytest
import torch

import hybrid_oracle as O

from drtc_amd import ops

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


def rnd(*shape, seed=0, dtype=F32, dev="cpu", std=1.0, mean=0.0):
    """Random values exact in ``dtype``, and the same in float64."""
    t = (torch.randn(*shape, generator=torch.Generator().manual_seed(seed)) * std + mean).to(dtype)
    return t.to(dev), t.double()


def i32(x, dev):
    return torch.as_tensor(np.asarray(x, np.int64), dtype=torch.int32, device=dev)


def portions(dev, lens, poss, slots):
    row = np.concatenate([[0], np.cumsum(lens)[:-1]])
    off = np.concatenate([np.arange(n) for n in lens])
    return ops.Portions(i32(row, dev), i32(lens, dev), i32(poss, dev), i32(slots, dev), i32(off, dev),
                        i32(np.repeat(slots, lens), dev), max(lens))


# ------------------------------------------------------------------ the stream
@on
@pytest.mark.parametrize("W", [256, 8, 100, 99, 520, 2048, 4096, 5120, 9216, 16384])
def test_layer_norm_behind_side_input(target, W):
    """The stream keeps 32 bits, the mean is taken off before the squares (a large common offset), y is
    normed before it is added, columns beyond the row are zero."""
    dev, dt = target
    rows = 5
    h, h64 = rnd(rows, W, seed=1, dev=dev, std=2, mean=30.0)
    y, y64 = rnd(rows, W + 8, seed=2, dtype=dt, dev=dev, std=5)
    yw, yw64 = rnd(W, seed=3, dev=dev)
    w, w64 = rnd(W, seed=4, dev=dev)
    want = h64 + O.rms(y64[:, :W], 1e-2) * yw64
    out = ops.side_norm(h, w, 1e-2, y[:, :W], yw, width=W + 24, dtype=dt)
    close(h, want, 1e-6)
    assert out.shape == (rows, W + 24) and (out[:, W:] == 0).all()
    close(out[:, :W], O.layer_norm(want, w64, 0.0, 1e-2), tol(dt, 2e-5, 5e-3))
    before = h.clone()
    close(ops.side_norm(h, w, 1e-2, dtype=dt), O.layer_norm(want, w64, 0.0, 1e-2), tol(dt, 2e-5, 5e-3))
    assert (before == h).all()
    e, e64 = rnd(11, W, seed=5, dtype=dt, dev=dev)
    ids = torch.arange(rows, dtype=torch.int32, device=dev) * 3 % 11
    out = ops.side_norm(h, w, 1e-5, ids=ids, embed=e, embed_scale=7.5, dtype=dt)
    close(h, e64[ids.long().cpu()] * 7.5, 1e-6)
    close(out, O.layer_norm(e64[ids.long().cpu()] * 7.5, w64, 0.0, 1e-5), tol(dt, 5e-6, 5e-3))


@on
@pytest.mark.parametrize("rows,W,dim", [(5, 256, 16), (1, 64, 7), (33, 100, 24), (300, 512, 128), (2, 99, 1), (17, 296, 40),
                                        (200, 128, 72), (600, 256, 32), (1, 2048, 128)])
def test_stream_add_and_side_gate(target, rows, W, dim):
    dev, dt = target
    h, h64 = rnd(rows, W, seed=1, dev=dev)
    y, y64 = rnd(rows, W, seed=2, dtype=dt, dev=dev)
    x = ops.stream_add(h, y)
    close(h, h64 + y64, 1e-6)
    close(x, h64 + y64, tol(dt, 1e-6, 5e-3))
    z, z64 = rnd(rows, dim, seed=3, dtype=dt, dev=dev, std=2)
    e, e64 = rnd(13, 3 * dim, seed=4, dtype=dt, dev=dev)
    ids = torch.arange(rows, dtype=torch.int32, device=dev) * 5 % 13
    for layer in range(3):
        want = O.gelu_tanh(z64) * e64[ids.long().cpu(), layer * dim:(layer + 1) * dim]
        close(ops.side_gate(z, e, ids, layer), want, tol(dt, 2e-6, 5e-3))
        w, w64 = rnd(dim, W, seed=5 + layer, dtype=dt, dev=dev, std=W ** -0.5)
        want = O.gelu_tanh(y64 @ w64.T) * e64[ids.long().cpu(), layer * dim:(layer + 1) * dim]
        close(ops.side_input(y, w, e, ids, layer), want, tol(dt, 2e-6, 1e-2))


# ------------------------------------------------------------------ retention and matrix memory
# heads, dim, vdim, rotated dims
SHAPES = [(2, 32, 48, 0), (3, 64, 64, 64), (2, 48, 32, 32), (1, 16, 8, 16), (2, 128, 128, 128), (2, 128, 200, 64),
          (1, 256, 256, 256), (1, 160, 72, 0), (2, 80, 400, 16), (1, 256, 520, 32), (3, 12, 20, 6), (2, 7, 9, 2),
          (1, 200, 261, 100), (2, 64, 30, 64)]


def memory(dev, dt, kind, shape, rows, seed=0, cap=8.0, eps=0.05, f_mean=3.0):
    """Random rows of the fused projection and layer operands.  ``eps`` lets the size of a read-out
    show through its norm; queries and keys share a direction, so that no read-out and no denominator
    is a small difference.  -> (proj, weights, float64 (q, k, v, i, f, gates, decay), states factory)."""
    H, d, dv, rot = shape
    pad = lambda n: -(-n // 8) * 8
    ok = pad(H * d)
    ov = ok + pad(H * d)
    og = ov + pad(H * dv)
    oi = og + pad(H * dv)
    of = oi + pad(H)
    proj, p64 = rnd(rows, of + pad(H) + 8, seed=seed, dtype=dt, dev=dev)
    for c in (0, ok):
        proj[:, c:c + H * d] += 0.7
    p64 = proj.double().cpu()
    base = 321.0
    w = ops.MemoryWeights(H, d, dv, eps, ok, ov, og, "silu" if kind == "retention" else "sigmoid")
    x = {"q": p64[:, :H * d].reshape(rows, H, d), "k": p64[:, ok:ok + H * d].reshape(rows, H, d),
         "v": p64[:, ov:ov + H * dv].reshape(rows, H, dv), "g": p64[:, og:og + H * dv], "base": base}
    if kind == "retention":
        decay = [1 - 2.0 ** (-1 - 6 * h / H) for h in range(H)]
        w.k_scale, w.rot_dims = d ** -0.5, rot
        w.rope = ops.build_interleaved_rope(1024, rot, base, dev) if rot else None
        w.log_decay = torch.tensor(decay, dtype=torch.float64).log().float().to(dev)
        x["decay"] = torch.tensor(decay, dtype=torch.float64)
    else:
        w.q_scale, w.off_i, w.off_f, w.cap = d ** -0.5, oi, of, cap
        w.i_bias, ib = rnd(H, seed=seed + 1, dev=dev, mean=1.0)
        w.f_bias, fb = rnd(H, seed=seed + 2, dev=dev, mean=f_mean)
        w.norm, x["norm"] = rnd(H * dv, seed=seed + 3, dev=dev, mean=1.0, std=0.3)
        proj[:, oi:oi + H] *= 3
        proj[:, of:of + H] *= 3
        x["i"] = (proj[:, oi:oi + H].double().cpu(), ib)
        x["f"] = (proj[:, of:of + H].double().cpu(), fb)

    def states(slots=5, fill=9.0):
        S = torch.full((slots, H, d, dv), fill, device=dev)
        if kind == "retention":
            return S, None, None
        n = ops.memory_slices(dv)
        return S, torch.full((slots, H, n, d), fill, device=dev), torch.full((slots, H, n), fill, device=dev)

    return proj, w, x, states


def expected(kind, shape, w, x, lo, hi):
    """Rows [lo, hi) as one whole sequence -> (outputs, final state)."""
    H, d, dv, rot = shape
    n, s = hi - lo, slice(lo, hi)
    pos = torch.arange(n)
    if kind == "retention":
        q = O.rotate_halves(x["q"][s], pos, x["base"], rot)
        k = O.rotate_halves(x["k"][s], pos, x["base"], rot) * d ** -0.5
        o, S = O.retention_scan(q, k, x["v"][s], x["decay"])
        return O.rms(o, w.eps).reshape(n, -1) * O.silu(x["g"][s]), (S,)
    i, f = (w.cap * torch.tanh((x[c][0][s] + x[c][1]) / w.cap) for c in "if")
    f = -torch.logaddexp(-f, torch.zeros_like(f))
    o, state = O.memory_scan(x["q"][s] * d ** -0.5, x["k"][s], x["v"][s], i, f)
    return O.rms(o, w.eps).reshape(n, -1) * x["norm"] * torch.sigmoid(x["g"][s]), state


def same_state(states, slot, want, t):
    """All copies of the slot's state; sizes differ by its running maximum's rounding."""
    close(states[0][slot], want[0], t)
    if states[1] is not None:
        for c in range(states[1].shape[2]):
            close(states[1][slot, :, c], want[1], t)
            close(states[2][slot, :, c], want[2], min(t, 1e-3))


@on
@pytest.mark.parametrize("kind", ["retention", "memory"])
@pytest.mark.parametrize("shape", SHAPES, ids=str)
@pytest.mark.parametrize("plain", [False, True])
def test_memory(target, kind, shape, plain):
    """Packed whole sequences, then one in portions and single decoded tokens, in state slots that hold
    another sequence's leftovers."""
    dev, dt = target
    if dev == "cpu" and plain:
        pytest.skip("one form")
    H, d, dv, _ = shape
    lens = [150, 1, 2, 64, 65]
    proj, w, x, fresh = memory(dev, dt, kind, shape, sum(lens))
    t = tol(dt, 1e-4, 3e-2)
    states, out = fresh(6), torch.full((sum(lens) + 1, H * dv + 8), 7.0, dtype=dt, device=dev)
    slots = [3, 0, 4, 1, 5]
    ops.memory_scan(proj, w, states, portions(dev, lens, [0] * 5, slots), out[:-1], plain=plain)
    assert (out[-1] == 7).all() and (out[:, H * dv:] == 7).all()
    a, wants = 0, []
    for n, s in zip(lens, slots):
        want, state = expected(kind, shape, w, x, a, a + n)
        wants.append(want)
        close(out[a:a + n, :H * dv], want, t)
        same_state(states, s, state, t)
        a += n
    assert all((s[2] == 9).all() for s in states if s is not None)

    # sequence 0 in portions and single tokens, a padding row beside
    states, a, rows = fresh(), 0, []
    for n in (2, 5, 1, 63, 2, 1, 1, 70, 5):
        x_ = proj[a:a + n + 1].contiguous()
        o = torch.full((n + 1, H * dv), 7.0, dtype=dt, device=dev)
        if n == 1:
            ops.memory_decode(x_, w, states, i32([a, 0], dev), i32([2, -1], dev), o)
        else:
            ops.memory_scan(x_, w, states, portions(dev, [n, 1], [a, 0], [2, -1]), o, plain=plain)
        assert (o[-1] == 0).all()
        rows.append(o[:-1])
        a += n
    assert a == 150
    close(torch.cat(rows), wants[0], t)
    same_state(states, 2, expected(kind, shape, w, x, 0, 150)[1], t)
    assert all((s[i] == 9).all() for s in states if s is not None for i in (0, 1, 3, 4))


@on
@pytest.mark.parametrize("kind", ["retention", "memory"])
def test_only_some_portions(target, kind):
    """The first portions of a step; the others' rows and slots stay."""
    dev, dt = target
    shape = (2, 32, 48, 32 if kind == "retention" else 0)
    proj, w, x, fresh = memory(dev, dt, kind, shape, 30)
    states, out = fresh(), torch.full((30, 96), 7.0, dtype=dt, device=dev)
    ops.memory_scan(proj, w, states, portions(dev, [20, 10], [0, 0], [1, 2]), out, portions=1)
    close(out[:20], expected(kind, shape, w, x, 0, 20)[0], tol(dt, 1e-4, 3e-2))
    assert (out[20:] == 7).all() and (states[0][2] == 9).all()


@on
@pytest.mark.parametrize("shape", [(2, 64, 64, 64), (1, 12, 20, 4)], ids=str)
@pytest.mark.parametrize("at,read", [(0, 299), (0, 63), (0, 64), (63, 64), (64, 127), (5, 6), (250, 250), (127, 256)])
def test_far_key_is_found_again(target, shape, at, read):
    """One loud key and value far back, a query that looks for it, at and beside chunk borders: it
    shows in a slowly decaying head, in prompts and when decoded."""
    dev, dt = target
    H, d, dv, rot = shape
    proj, w, x, fresh = memory(dev, dt, "retention", shape, 300)
    w.log_decay.fill_(float(np.log(0.9995)))
    x["decay"].fill_(0.9995)
    key = torch.sign(x["k"][at]) * 4
    # turned back, so that both meet in the same phase
    back = O.rotate_halves(key[None], torch.tensor([at - read]), x["base"], rot)[0].to(dt)
    proj[at, w.off_k:w.off_k + H * d] = key.flatten().to(dt).to(dev)
    proj[read, :H * d] = back.flatten().to(dev)
    proj[at, w.off_v:w.off_v + H * dv] = 8 * torch.sign(proj[at, w.off_v:w.off_v + H * dv])
    x["k"][at], x["q"][read] = key, back.double()
    x["v"][at] = proj[at, w.off_v:w.off_v + H * dv].double().cpu().reshape(H, dv)
    want = expected("retention", shape, w, x, 0, read + 1)[0][read]
    x["v"][at] *= -1
    other = expected("retention", shape, w, x, 0, read + 1)[0][read]
    assert (want - other).abs().max() > 1  # the key shows in what is expected
    for cut in (0, read - 1, read):  # whole, a portion of two, decoded
        states, a = fresh(), 0
        for n in (cut, read + 1 - cut):
            if n > 1 or (n == 1 and a == 0):
                o = torch.empty(n, H * dv, dtype=dt, device=dev)
                ops.memory_scan(proj[a:a + n].contiguous(), w, states, portions(dev, [n], [a], [2]), o)
            elif n == 1:
                o = torch.empty(1, H * dv, dtype=dt, device=dev)
                ops.memory_decode(proj[a:a + 1].contiguous(), w, states, i32([a], dev), i32([2], dev), o)
            a += n
        close(o[-1], want, tol(dt, 1e-4, 3e-2))


@on
@pytest.mark.parametrize("cap,i_mean,f_mean", [(2.0, 30.0, 30.0), (40.0, 38.0, 20.0), (12.0, -40.0, 40.0),
                                               (15.0, 0.0, -40.0), (6.0, 4.0, 4.0), (25.0, -10.0, 12.0)])
def test_gates_at_their_caps(target, cap, i_mean, f_mean):
    """Gates pinned to either cap: large running maxima (the 1e-6 of the denominator counts), inputs
    that never exceed the start of the maximum, memories that forget everything at once."""
    dev, dt = target
    shape = (2, 32, 48, 0)
    proj, w, x, fresh = memory(dev, dt, "memory", shape, 200, cap=cap, eps=1e-4)
    for c, b, mean in (("i", w.i_bias, i_mean), ("f", w.f_bias, f_mean)):
        b += mean
        x[c] = (x[c][0], b.double().cpu())
    want, state = expected("memory", shape, w, x, 0, 200)
    for plain in (False, True):
        states, o = fresh(), torch.empty(200, 96, dtype=dt, device=dev)
        ops.memory_scan(proj[:130].contiguous(), w, states, portions(dev, [130], [0], [1]), o[:130], plain=plain)
        ops.memory_decode(proj[130:131].contiguous(), w, states, i32([130], dev), i32([1], dev), o[130:131])
        ops.memory_scan(proj[131:].contiguous(), w, states, portions(dev, [69], [131], [1]), o[131:], plain=plain)
        assert not torch.isnan(o).any()
        close(o, want, tol(dt, 2e-4, 3e-2))
        same_state(states, 1, state, tol(dt, 2e-4, 3e-2))


@on
def test_denominator_counts(target):
    """Its two branches and what is added to them, seen through a norm whose eps dominates."""
    dev, dt = target
    shape = (1, 32, 32, 0)
    proj, w, x, fresh = memory(dev, dt, "memory", shape, 90, cap=14.0, eps=1e3, f_mean=6.0)
    proj[:10, w.off_i] = x["i"][0][:10] = -30  # hardly written at first: the other branch
    want, _ = expected("memory", shape, w, x, 0, 90)
    states, o = fresh(), torch.empty(90, 32, dtype=dt, device=dev)
    ops.memory_scan(proj, w, states, portions(dev, [90], [0], [1]), o)
    for rows in (slice(0, 10), slice(10, 90)):
        d = (o.double().cpu() - want)[rows].abs().amax(0)
        assert (d <= tol(dt, 1e-4, 2e-2) * want[rows].abs().amax(0)).all()
    # the branches differ by orders of magnitude
    assert want[10:].abs().mean() > 30 * want[:10].abs().mean()


# ------------------------------------------------------------------ latent attention
@on
@pytest.mark.parametrize("dims", [(3, 24, 8, 40), (2, 128, 64, 128), (1, 160, 64, 200), (2, 12, 6, 21)], ids=str)
def test_head_gates_of_prompts(target, dims):
    """Outputs times the sigmoid of a gate per head and row."""
    dev, dt = target
    H, dim, rot, vdim = dims
    R, lens, ctx = 16, [70, 2, 131], [0, 90, 33]
    voff = -(-H * dim // 8) * 8
    n, K = sum(lens), sum(lens) + sum(ctx)
    q, _ = rnd(n, H * (dim + rot), seed=1, dtype=dt, dev=dev)
    kv, _ = rnd(K, voff + -(-H * vdim // 8) * 8, seed=2, dtype=dt, dev=dev)
    lat, _ = rnd(K, ops.latent_width(R, rot), seed=3, dtype=dt, dev=dev)
    gate, g64 = rnd(n, H + 3, seed=4, dtype=dt, dev=dev, std=2)
    q_cu = np.concatenate([[0], np.cumsum(lens)])
    k_cu = np.concatenate([[0], np.cumsum(np.add(lens, ctx))])
    qt = ops.latent_qtile(max(lens), dim, rot, vdim)
    tiles = tuple(i32(t, dev) for t in ops.portion_tiles(q_cu.tolist(), qt))
    keys = ops.PortionKeys(i32(k_cu, dev), i32(ctx, dev), None, k_cu.tolist(), ctx)
    outs = []
    for g in (None, gate[:, :H]):
        o = torch.full((n, H * vdim + 8), 5.0, dtype=dt, device=dev)
        ops.latent_prefill_attention(q, kv, voff, lat, R, H, dim, rot, vdim, i32(q_cu, dev), q_cu.tolist(), keys,
                                     tiles, qt, None, 0.1, None, o[:, :H * vdim], g)
        assert (o[:, H * vdim:] == 5).all()
        outs.append(o[:, :H * vdim].double().cpu().reshape(n, H, vdim))
    close(outs[1], outs[0] * torch.sigmoid(g64[:, :H, None]), tol(dt, 1e-5, 1e-2))


@on
@pytest.mark.parametrize("H,R,rot", [(4, 48, 16), (20, 160, 32), (3, 52, 6)])
def test_head_gates_of_decoded_tokens(target, H, R, rot):
    dev, dt = target
    LW, nb = ops.latent_width(R, rot), 6
    ctx = [1, 33, 64, 190, 0]
    B = len(ctx)
    cache, _ = rnd(B * nb + 1, 32, LW, seed=1, dtype=dt, dev=dev, std=0.7)
    cache[..., R + rot:] = 0
    bt = (torch.arange(B * nb).view(B, nb).to(torch.int32) + 1).to(dev)
    qa, _ = rnd(B, H, LW, seed=2, dtype=dt, dev=dev, std=0.5)
    gate, g64 = rnd(B, H + 1, seed=3, dtype=dt, dev=dev, std=2)
    for parts in (1, 3):
        outs = []
        for g in (None, gate[:, :H]):
            ws = None
            if dev == "cuda":
                ws = ops.LatentDecodeWorkspace(B, H, R, None, nb, dev)
                ws.per, ws.splits = -(-nb // parts), parts
                ws.part_o = torch.empty(B, H, parts, R, device=dev)
                ws.part_ml = torch.empty(B, H, parts, 2, device=dev)
            outs.append(ops.latent_decode_attention(qa, cache, R, bt, i32(ctx, dev), None, 0.11, None, ws, g))
        close(outs[1], outs[0].double().cpu() * torch.sigmoid(g64[:, :H, None]), tol(dt, 1e-5, 1e-2))
        assert (outs[1][-1] == 0).all()


@on
@pytest.mark.parametrize("rot", [16, 6])
def test_queries_without_latents(target, rot):
    """A layer that reads another one's rows turns its queries and leaves the cache alone."""
    dev, dt = target
    H, dim, R, n = 3, 16, 40, 5
    LW = ops.latent_width(R, rot)
    proj, p64 = rnd(n, H * (dim + rot), seed=1, dtype=dt, dev=dev)
    pos = torch.tensor([0, 1, 31, 700, 1023], dtype=torch.int32)
    cache = torch.full((2, 32, LW), 7.0, dtype=dt, device=dev)
    qa = torch.full((n, H, LW), 3.0, dtype=dt, device=dev)
    cs = ops.build_interleaved_rope(1024, rot, 321.0, dev)
    args = (None, H, dim, rot, rot, R, None, 1e-5, cs, pos.to(dev), torch.arange(n, device=dev), cache)
    ops.latent_prep(proj, *args, qa=qa)
    ops.latent_prep(proj, *args)
    q = O.rotate_interleaved(p64.reshape(n, H, -1)[..., dim:], pos, 321.0, rot)
    close(proj.reshape(n, H, -1)[..., dim:], q, tol(dt, 1e-5, 1e-2))
    close(proj.reshape(n, H, -1)[..., :dim], p64.reshape(n, H, -1)[..., :dim], 0)
    close(qa[..., R:R + rot], q, tol(dt, 1e-5, 1e-2))
    assert (qa[..., R + rot:] == 0).all() and (qa[..., :R] == 3).all() and (cache == 7).all()


# ------------------------------------------------------------------ experts
@on
@pytest.mark.parametrize("T,W,ff,E,top", [(1, 256, 128, 8, 2), (37, 128, 128, 5, 5), (300, 256, 256, 4, 2),
                                          (1500, 256, 256, 4, 2), (64, 512, 384, 16, 4), (700, 384, 128, 6, 1),
                                          (260, 256, 256, 1, 1), (129, 256, 640, 3, 2)])
@pytest.mark.parametrize("stream", [False, True])
def test_squared_relu_experts(target, T, W, ff, E, top, stream):
    """No gate: relu(up)^2; alone, or added to the 32-bit stream beside another sublayer's output (fewer
    columns than the experts have)."""
    dev, dt = target
    x, x64 = rnd(T, W, seed=1, dtype=dt, dev=dev)
    r, r64 = rnd(E, W, seed=2, dtype=dt, dev=dev, std=6 * W ** -0.5)
    up, u64 = rnd(E, ff, W, seed=3, dtype=dt, dev=dev, std=W ** -0.5)
    dn, d64 = rnd(E, W, ff, seed=4, dtype=dt, dev=dev, std=ff ** -0.5)
    Wt = {"router": r64, **{f"e{e}.up": u64[e] for e in range(E)}, **{f"e{e}.down": d64[e] for e in range(E)}}
    mlp = {"router": {"experts": E, "top": top}}
    want = O.relu2_experts(x64, Wt, mlp)
    sure = O.route_margin(x64, r64, mlp["router"]) > 1e-3
    t = tol(dt, 2e-5, 2e-2)
    logits = ops.router_logits_f32(x, r)
    if dev == "cuda":
        # large steps and small ones take different kernels; each where it takes the sizes
        variants = [None] if dt == F32 else [None, 0, 1, 2] + ([4] if ff % 256 == 0 and W % 256 == 0 else []) + \
            ([3] if ff >= 512 and W >= 512 else [])
    else:
        variants = [None]
    for v in variants:
        if not stream:
            got = ops.fused_moe(x, logits, up, dn, top, "relu2", variant=v)
            close(got[sure.to(dev)], want[sure], t)
            continue
        for n in (W, W - 8, W - 3):
            h, h64 = rnd(T, n, seed=5, dev=dev, std=2)
            y, y64 = rnd(T, n + 8, seed=6, dtype=dt, dev=dev)
            got = ops.fused_moe(x, logits, up, dn, top, "relu2", variant=v, stream=h, y=y[:, :n])
            both = (h64 + want[:, :n] + y64[:, :n])[sure]
            close(h[sure.to(dev)], both, tol(dt, 2e-5, 1e-2))
            close(got[sure.to(dev)], both, t)


@pytest.mark.gpu
def test_experts_on_wide_tiles():
    """The XCD-partitioned grouped GEMM (about a tile of rows to an expert)."""
    T, W, ff, E, top = 900, 1024, 512, 6, 1
    x, x64 = rnd(T, W, seed=1, dtype=BF16, dev="cuda")
    r, r64 = rnd(E, W, seed=2, dtype=BF16, dev="cuda", std=6 * W ** -0.5)
    up, u64 = rnd(E, ff, W, seed=3, dtype=BF16, dev="cuda", std=W ** -0.5)
    dn, d64 = rnd(E, W, ff, seed=4, dtype=BF16, dev="cuda", std=ff ** -0.5)
    Wt = {"router": r64, **{f"e{e}.up": u64[e] for e in range(E)}, **{f"e{e}.down": d64[e] for e in range(E)}}
    mlp = {"router": {"experts": E, "top": top}}
    sure = O.route_margin(x64, r64, mlp["router"]) > 1e-3
    want = O.relu2_experts(x64, Wt, mlp)[sure]
    for v in (None, 1, 2, 3, 4):
        got = ops.fused_moe(x, ops.router_logits_f32(x, r), up, dn, top, "relu2", variant=v)
        close(got[sure.to("cuda")], want, 2e-2)


@pytest.mark.gpu
@pytest.mark.parametrize("form", [121, 141, 142, 161, 241, 261, 281])
def test_squared_relu_on_xcd_tiles(form):
    """The epilogue of the XCD-partitioned GEMM, into columns of a wider operand."""
    M, N, K = 200, 768, 768
    x, x64 = rnd(M, K, seed=1, dtype=BF16, dev="cuda")
    w, w64 = rnd(N, K, seed=2, dtype=BF16, dev="cuda", std=K ** -0.5)
    a = torch.full((M, 8 + N + 8), 5.0, dtype=BF16, device="cuda")
    ops.gemm.xd_gemm(x, w, "relu2", out=a[:, 8:8 + N], form=form)
    close(a[:, 8:8 + N], torch.relu(x64 @ w64.T).square(), 1e-2)
    assert (a[:, :8] == 5).all() and (a[:, 8 + N:] == 5).all()
