"""Latent attention over a paged cache of per-token latents.

HIP kernels: csrc/kernels/latent_attention.hip.  A cache row holds a token's normed latent
(``kv_rank``), the rotated key part all heads share (``rot_dim``) and zeros up to a multiple of
32 columns (``latent_width``).  Prompt portions attend with per-head keys and values projected
up from the latents; decode rows project the query down instead and attend to the cached rows
themselves (``head_linear`` before and after).
"""
from __future__ import annotations

import math
from dataclasses import dataclass

import torch

from ._ext import check, hipk, on_gpu, ptr, stream_ptr
from .attention import KV_BLOCK


def latent_width(kv_rank: int, rot_dim: int) -> int:
    return -(-(kv_rank + rot_dim) // 32) * 32


def build_interleaved_rope(max_pos: int, dims: int, base: float, device=None,
                           scaling=None) -> torch.Tensor:
    """[max_pos, dims] fp32: cos then sin of position * base^(-2i / dims), i < dims / 2.

    ``scaling`` (models.config.RotaryScaling), for contexts ``factor`` times the ``original`` one:
    pairs that turn more than ``fast`` times within the original context keep their speed, those
    that turn less than ``slow`` times are slowed down by the factor, the ones between are blended
    along the pair index, and cosine and sine grow by 0.1 ln(factor) + 1."""
    i = torch.arange(dims // 2, dtype=torch.float64)
    inv = base ** (-2.0 * i / dims)
    mag = 1.0
    if scaling is not None:
        def pair(turns):  # the (fractional) pair that turns so often within the original context
            return dims * math.log(scaling.original / (2 * math.pi * turns)) / (2 * math.log(base))

        lo = max(math.floor(pair(scaling.fast)), 0)
        hi = min(math.ceil(pair(scaling.slow)), dims - 1)
        slowed = ((i - lo) / max(hi - lo, 0.001)).clamp(0, 1)
        inv = inv * (slowed / scaling.factor + 1 - slowed)
        mag = 0.1 * math.log(scaling.factor) + 1
    ang = torch.outer(torch.arange(max_pos, dtype=torch.float64), inv)
    return (torch.cat([torch.cos(ang), torch.sin(ang)], -1) * mag).to(torch.float32).to(device or "cpu")


def rotate_pairs_ref(x: torch.Tensor, cs: torch.Tensor, dims: int) -> torch.Tensor:
    """Rotate pairs (2i, 2i+1) of x's first ``dims`` components; cs [rows, dims] broadcast over
    the axes between."""
    half = dims // 2
    c = cs[:, :half].reshape(x.shape[0], *([1] * (x.dim() - 2)), half)
    s = cs[:, half:].reshape(c.shape)
    xf = x.float()
    out = xf.clone()
    u, v = xf[..., 0:dims:2], xf[..., 1:dims:2]
    out[..., 0:dims:2] = u * c - v * s
    out[..., 1:dims:2] = v * c + u * s
    return out.to(x.dtype)


# ------------------------------------------------------------------ per-token preparation
def latent_prep(proj: torch.Tensor, off_kv: int | None, heads: int, dim: int, rot_dim: int,
                rot_dims: int, kv_rank: int, norm_w: torch.Tensor | None, eps: float,
                cos_sin: torch.Tensor, positions: torch.Tensor, slots: torch.Tensor | None,
                cache: torch.Tensor | None, lat: torch.Tensor | None = None,
                qa: torch.Tensor | None = None) -> None:
    """Rows of the fused projection [queries | latent, key part]: RMS-norm the latent, rotate
    the key part, write both to ``lat`` [rows, LW] and to the cache rows ``slots`` (-1: none).
    The queries' rotated parts go to ``qa`` [rows, heads, LW] at column kv_rank (zeros
    behind), or are rotated in place.  ``off_kv`` None: queries only."""
    rows = proj.shape[0]
    own = off_kv is not None
    LW = (cache if cache is not None else lat if lat is not None else qa).shape[-1]
    dq = dim + rot_dim
    if not on_gpu(proj):
        cs = cos_sin[positions[:rows].long()]
        if own:
            kv = proj[:, off_kv:off_kv + kv_rank + rot_dim]
            cf = kv[:, :kv_rank].float()
            c = cf * torch.rsqrt(cf.pow(2).mean(-1, keepdim=True) + eps) * norm_w
            full = proj.new_zeros(rows, LW)
            full[:, :kv_rank] = c.to(proj.dtype)
            full[:, kv_rank:kv_rank + rot_dim] = rotate_pairs_ref(kv[:, kv_rank:], cs, rot_dims)
            if lat is not None:
                lat.copy_(full)
            if cache is not None and slots is not None:
                ok = slots[:rows] >= 0
                cache.view(-1, LW)[slots[:rows][ok]] = full[ok]
        q = proj[:, :heads * dq].unflatten(1, (heads, dq))
        r = rotate_pairs_ref(q[..., dim:], cs, rot_dims)
        if qa is not None:
            qa[..., kv_rank:] = 0
            qa[..., kv_rank:kv_rank + rot_dim] = r
        else:
            q[..., dim:] = r
        return
    assert proj.dim() == 2 and proj.stride(1) == 1
    assert heads * dq <= (off_kv if own else proj.shape[1])
    assert not own or off_kv + kv_rank + rot_dim <= proj.shape[1]
    assert positions.dtype == torch.int32 and positions.numel() >= rows
    assert cos_sin.dtype == torch.float32 and cos_sin.shape[1] == rot_dims
    assert cos_sin.is_contiguous()
    assert not own or (norm_w.dtype == torch.float32 and norm_w.numel() == kv_rank)
    for t in (lat, cache, qa):
        assert t is None or (t.is_contiguous() and t.shape[-1] == LW and t.dtype == proj.dtype)
    assert lat is None or lat.shape[0] == rows
    assert qa is None or qa.shape[:2] == (rows, heads)
    if cache is not None:
        assert slots is not None and slots.dtype == torch.int64 and slots.numel() >= rows
    check(hipk().latent_prep(int(proj.dtype == torch.float32), dict(
        proj=proj.data_ptr(), ldp=proj.stride(0), off_kv=off_kv if own else -1, H=heads, dim=dim,
        rot=rot_dim, rot_dims=rot_dims, R=kv_rank, LW=LW, norm_w=ptr(norm_w), eps=float(eps),
        cos_sin=cos_sin.data_ptr(), positions=positions.data_ptr(), slots=ptr(slots),
        lat=ptr(lat), cache=ptr(cache), qa=ptr(qa), rows=rows), stream_ptr(proj)), "latent_prep")


def latent_gather(cache: torch.Tensor, slots: torch.Tensor) -> torch.Tensor:
    """Cache rows of ``slots`` (int64, -1: a zero row) -> [n, LW]."""
    LW = cache.shape[-1]
    if not on_gpu(cache):
        out = cache.view(-1, LW)[slots.clamp(min=0)]
        out[slots < 0] = 0
        return out
    assert slots.dtype == torch.int64 and slots.is_cuda and cache.is_contiguous()
    out = torch.empty((slots.numel(), LW), dtype=cache.dtype, device=cache.device)
    check(hipk().latent_gather(out.data_ptr(), cache.data_ptr(), slots.data_ptr(), slots.numel(),
                               LW * cache.element_size(), stream_ptr(cache)), "latent_gather")
    return out


# ------------------------------------------------------------------ prompt portions
@dataclass
class PortionKeys:
    """Key rows of a packed set of prompt portions under one window: the tokens of each
    portion and the window's reach ahead of it.  ``slots`` None: no portion has anything
    ahead, the key rows are the portions' own rows."""
    k_cu: torch.Tensor           # int32 [n + 1]
    ctx: torch.Tensor            # int32 [n]: key rows ahead of the portion's first token
    slots: torch.Tensor | None   # int64 [keys]: cache rows
    k_host: list
    ctx_host: list


def window_reach(start: int, window: int | None) -> int:
    """Cached tokens a portion starting at ``start`` can see ahead of its first token."""
    return start if window is None else min(start, window - 1)


def latent_qtile(max_len: int, dim: int, rot_dim: int, vdim: int) -> int:
    """Query rows per workgroup (64: one 16-row fragment a wave; 128 / 256: two, where the sizes
    leave registers for them), by the longest portion."""
    if dim + rot_dim > 192 or vdim > 128 or max_len <= 64:
        return 64
    return 128 if max_len < QTILE_256_MIN else 256


QTILE_256_MIN = 192


def portion_tiles(cu: list[int], qtile: int) -> tuple[list[int], list[int]]:
    """(portion, first query row in it) of every query tile, longest portions first."""
    order = sorted(range(len(cu) - 1), key=lambda s: cu[s] - cu[s + 1])
    ts, tq = [], []
    for s in order:
        for q0 in range(0, cu[s + 1] - cu[s], qtile):
            ts.append(s)
            tq.append(q0)
    return ts, tq


def latent_prefill_attention(q: torch.Tensor, kv: torch.Tensor, voff: int, lat: torch.Tensor,
                             kv_rank: int, heads: int, dim: int, rot_dim: int, vdim: int,
                             q_cu: torch.Tensor, q_host: list, keys: PortionKeys,
                             tiles: tuple, qtile: int, window: int | None, scale: float,
                             sink: torch.Tensor | None, out: torch.Tensor,
                             gate: torch.Tensor | None = None) -> torch.Tensor:
    """Causal windowed attention of packed prompt portions.  q rows: heads of [dim | rotated];
    kv rows: per-head keys [heads * dim], values from column ``voff``; lat rows: the shared
    rotated key part from column kv_rank.  ``gate`` [rows, heads]: outputs times its sigmoid.
    Writes out[:q_host[-1]] ([rows, heads * vdim])."""
    if not on_gpu(q):
        return _latent_prefill_ref(q, kv, voff, lat, kv_rank, heads, dim, rot_dim, vdim, q_host,
                                   keys, window, scale, sink, out, gate)
    n = len(q_host) - 1
    for t in (q, kv, lat, out):
        assert t.stride(1) == 1 and t.dtype == q.dtype and t.is_cuda
    assert q.shape[0] >= q_host[-1] and out.shape[0] >= q_host[-1]
    assert kv.shape[0] >= keys.k_host[-1] and lat.shape[0] >= keys.k_host[-1]
    assert kv.shape[1] >= voff + heads * vdim and out.shape[1] >= heads * vdim
    assert q.shape[1] >= heads * (dim + rot_dim) and lat.stride(0) == lat.shape[1]
    assert sink is None or (sink.dtype == torch.float32 and sink.numel() == heads)
    _check_gate(gate, q, q_host[-1], heads)
    for t in (q_cu, keys.k_cu, keys.ctx, *tiles):
        assert t.dtype == torch.int32 and t.is_cuda
    assert q_cu.numel() == n + 1 and keys.k_cu.numel() == n + 1 and keys.ctx.numel() == n
    check(hipk().latent_prefill(int(q.dtype == torch.float32), dict(
        out=out.data_ptr(), ldo=out.stride(0), q=q.data_ptr(), ldq=q.stride(0), kv=kv.data_ptr(),
        ldkv=kv.stride(0), voff=voff, lat=lat.data_ptr(), LW=lat.shape[1], R=kv_rank, H=heads,
        dim=dim, rot=rot_dim, vdim=vdim, q_cu=q_cu.data_ptr(), k_cu=keys.k_cu.data_ptr(),
        ctx=keys.ctx.data_ptr(), tile_seq=tiles[0].data_ptr(), tile_q0=tiles[1].data_ptr(),
        ntiles=tiles[0].numel(), qtile=qtile, nseq=n, nq=q_host[-1], window=window or 0,
        scale=float(scale), sink=ptr(sink), gate=ptr(gate),
        ldg=gate.stride(0) if gate is not None else 0), stream_ptr(q)), "latent_prefill")
    return out


def _check_gate(gate, x, rows: int, heads: int) -> None:
    assert gate is None or (gate.dtype == x.dtype and gate.stride(1) == 1 and gate.is_cuda
                            and gate.shape[0] >= rows and gate.shape[1] == heads)


def _sink_softmax_ref(sc: torch.Tensor, sink: torch.Tensor | None) -> torch.Tensor:
    """Softmax over the last axis of sc [heads, ...], a per-head term in the denominator."""
    if sink is None:
        return torch.softmax(sc, dim=-1)
    extra = sink.view(-1, *([1] * (sc.dim() - 1))).expand(*sc.shape[:-1], 1)
    return torch.softmax(torch.cat([sc, extra], -1), dim=-1)[..., :-1]


def _latent_prefill_ref(q, kv, voff, lat, kv_rank, heads, dim, rot_dim, vdim, q_host, keys,
                        window, scale, sink, out, gate=None):
    dq = dim + rot_dim
    for s, ctx in enumerate(keys.ctx_host):
        a, b = q_host[s], q_host[s + 1]
        k0, k1 = keys.k_host[s], keys.k_host[s + 1]
        qs = q[a:b, :heads * dq].float().unflatten(1, (heads, dq))
        kn = kv[k0:k1, :heads * dim].float().unflatten(1, (heads, dim))
        v = kv[k0:k1, voff:voff + heads * vdim].float().unflatten(1, (heads, vdim))
        kr = lat[k0:k1, kv_rank:kv_rank + rot_dim].float()
        sc = (torch.einsum("ihd,jhd->hij", qs[..., :dim], kn)
              + torch.einsum("ihr,jr->hij", qs[..., dim:], kr)) * scale
        d = (torch.arange(b - a)[:, None] + ctx) - torch.arange(k1 - k0)[None, :]
        hide = d < 0 if window is None else (d < 0) | (d >= window)
        p = _sink_softmax_ref(sc.masked_fill(hide.to(sc.device), float("-inf")), sink)
        o = torch.einsum("hij,jhv->ihv", p, v)
        if gate is not None:
            o = o * torch.sigmoid(gate[a:b].float())[..., None]
        out[a:b, :heads * vdim] = o.flatten(1).to(out.dtype)
    return out


# ------------------------------------------------------------------ decode rows
def latent_decode_splits(batch: int, heads: int, window: int | None, max_blocks: int,
                         target_wgs: int = 256) -> tuple[int, int]:
    """(cache blocks per split, splits): static, so that a decode step can be captured.  Splits
    fill the chip when the batch alone does not; at least 4 blocks each."""
    blocks = max_blocks if window is None else min(max_blocks, (window + KV_BLOCK - 2) // KV_BLOCK + 1)
    groups = -(-heads // 64)
    want = max(1, target_wgs // max(1, batch * groups))
    per = max(4, -(-blocks // want))
    return per, -(-blocks // per)


class LatentDecodeWorkspace:
    """fp32 partials of the split window, one per (batch bucket, layer geometry)."""

    def __init__(self, batch: int, heads: int, kv_rank: int, window: int | None, max_blocks: int,
                 device):
        self.per, self.splits = latent_decode_splits(batch, heads, window, max_blocks)
        self.part_o = self.part_ml = None
        if self.splits > 1 and torch.device(device).type == "cuda":
            self.part_o = torch.empty((batch, heads, self.splits, kv_rank), dtype=torch.float32,
                                      device=device)
            self.part_ml = torch.empty((batch, heads, self.splits, 2), dtype=torch.float32,
                                       device=device)


def latent_decode_attention(qa: torch.Tensor, cache: torch.Tensor, kv_rank: int,
                            block_tables: torch.Tensor, context_lens: torch.Tensor,
                            window: int | None, scale: float, sink: torch.Tensor | None,
                            workspace: LatentDecodeWorkspace | None = None,
                            gate: torch.Tensor | None = None) -> torch.Tensor:
    """One query per sequence in the latent space, qa [B, heads, LW], against the cache rows of
    its last ``window`` tokens (its own included: context_lens counts it).  Rows with context 0
    give zeros.  ``gate`` [B, heads]: results times its sigmoid.  Returns [B, heads, kv_rank]."""
    B, H, LW = qa.shape
    if not on_gpu(qa):
        out = qa.new_zeros(B, H, kv_rank)
        flat = cache.view(-1, LW)
        for b in range(B):
            n = int(context_lens[b])
            if n <= 0:
                continue
            j = torch.arange(0 if window is None else max(0, n - window), n, device=qa.device)
            rows = flat[block_tables[b].long()[j // KV_BLOCK] * KV_BLOCK + j % KV_BLOCK].float()
            p = _sink_softmax_ref(qa[b].float() @ rows.T * scale, sink)
            o = p @ rows[:, :kv_rank]
            if gate is not None:
                o = o * torch.sigmoid(gate[b].float())[:, None]
            out[b] = o.to(out.dtype)
        return out
    assert qa.is_contiguous() and cache.is_contiguous() and cache.shape[1:] == (KV_BLOCK, LW)
    assert cache.dtype == qa.dtype and block_tables.dtype == torch.int32
    assert block_tables.stride(1) == 1 and block_tables.shape[0] >= B
    assert context_lens.dtype == torch.int32 and context_lens.numel() >= B
    assert sink is None or (sink.dtype == torch.float32 and sink.numel() == H)
    _check_gate(gate, qa, B, H)
    ws = workspace or LatentDecodeWorkspace(B, H, kv_rank, window, block_tables.shape[1], qa.device)
    assert ws.splits == 1 or (ws.part_o is not None and ws.part_o.shape[:2] == (B, H)
                              and ws.part_o.shape[3] == kv_rank)
    out = torch.empty((B, H, kv_rank), dtype=qa.dtype, device=qa.device)
    check(hipk().latent_decode(int(qa.dtype == torch.float32), dict(
        out=out.data_ptr(), part_o=ptr(ws.part_o), part_ml=ptr(ws.part_ml), qa=qa.data_ptr(),
        cache=cache.data_ptr(), block_tables=block_tables.data_ptr(),
        bt_stride=block_tables.stride(0), context_lens=context_lens.data_ptr(), B=B, H=H,
        R=kv_rank, LW=LW, window=window or 0, tiles_per_split=ws.per, nsplits=ws.splits,
        scale=float(scale), sink=ptr(sink), gate=ptr(gate),
        ldg=gate.stride(0) if gate is not None else 0), stream_ptr(qa)), "latent_decode")
    return out


def head_linear(x: torch.Tensor, w: torch.Tensor, out: torch.Tensor | None = None) -> torch.Tensor:
    """y[b, h] = w[h] @ x[b, h]: x [B, H, >= K] (any batch / head stride), w [H, N, K],
    out [B, H, >= N] view written in its first N columns."""
    B, H = x.shape[:2]
    N, K = w.shape[1:]
    if out is None:
        out = x.new_empty(B, H, N)
    if not on_gpu(x):
        out[..., :N] = torch.einsum("bhk,hnk->bhn", x[..., :K].float(), w.float()).to(out.dtype)
        return out
    assert x.stride(2) == 1 and out.stride(2) == 1 and w.is_contiguous() and w.shape[0] == H
    assert x.shape[2] >= K and out.shape[2] >= N and x.dtype == w.dtype == out.dtype
    check(hipk().head_gemm(int(x.dtype == torch.float32), out.data_ptr(), x.data_ptr(),
                           w.data_ptr(), B, H, N, K, out.stride(0), out.stride(1), x.stride(0),
                           x.stride(1), stream_ptr(x)), "head_gemm")
    return out

