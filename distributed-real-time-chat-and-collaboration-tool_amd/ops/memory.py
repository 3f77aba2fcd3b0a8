"""Linear attention with a matrix state per head, S <- a S + b k v^T, read out with the query:
retention (a fixed decay a, b = 1) and the mLSTM (exponential input and sigmoid forget gates, a
normaliser and a running maximum).

HIP kernels: csrc/kernels/memory_scan.hip.  One kernel family takes both: with log gates f, i and
m_t = max(f_t + m_(t-1), i_t) from m = 0 on, a = e^(f + m_(t-1) - m_t) and b = e^(i - m_t), so a
retention layer is f = log decay, i = 0, where m stays 0.  Each head's read-out is divided by its
root mean square, weighted, gated and handed to the output projection.

A sequence's state (32-bit) is addressed by the state slot its rows carry; slot -1 marks padding
rows, position 0 starts from zero whatever the slot held.
"""
from __future__ import annotations

from dataclasses import dataclass

import torch
import torch.nn.functional as F

from ._ext import check, hipk, on_gpu, ptr, stream_ptr
from .delta import Portions

SLICE_COLUMNS = 128  # a workgroup's value columns


def memory_slices(vdim: int) -> int:
    """Workgroups a head's columns are split over; each keeps its own copy of the normaliser and the
    running maximum."""
    return -(-vdim // SLICE_COLUMNS)


@dataclass
class MemoryWeights:
    """Small per-layer operands (32-bit) and where the fused projection [queries | ... ] holds the
    keys, values, read-out gates and (mLSTM) gate inputs."""
    heads: int
    dim: int
    vdim: int
    eps: float
    off_k: int
    off_v: int
    off_g: int
    act: str                             # of the read-out gate: "silu" or "sigmoid"
    q_scale: float = 1.0
    k_scale: float = 1.0
    rope: torch.Tensor | None = None     # [positions, rot_dims] cos | sin
    rot_dims: int = 0
    log_decay: torch.Tensor | None = None  # [heads] retention
    off_i: int = 0
    off_f: int = 0
    i_bias: torch.Tensor | None = None   # [heads] mLSTM
    f_bias: torch.Tensor | None = None
    cap: float = 0.0
    norm: torch.Tensor | None = None     # [heads * vdim]

    @property
    def gated(self) -> bool:
        return self.log_decay is None


def rotate_halves_ref(x: torch.Tensor, cs: torch.Tensor, dims: int) -> torch.Tensor:
    """Rotate components i, i + dims / 2 of x [rows, heads, D]; cs [rows, dims]."""
    half = dims // 2
    c, s = cs[:, None, :half], cs[:, None, half:]
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., dims:]], -1)


def _rows_ref(proj, w: MemoryWeights, positions):
    n, H, kd, vd = proj.shape[0], w.heads, w.heads * w.dim, w.heads * w.vdim
    x = proj.float()
    q, k = x[:, :kd].reshape(n, H, w.dim), x[:, w.off_k:w.off_k + kd].reshape(n, H, w.dim)
    if w.rot_dims:
        cs = w.rope[positions[:n].long()]
        q, k = (rotate_halves_ref(t, cs, w.rot_dims) for t in (q, k))
    if w.gated:
        i = w.cap * torch.tanh((x[:, w.off_i:w.off_i + H] + w.i_bias) / w.cap)
        f = F.logsigmoid(w.cap * torch.tanh((x[:, w.off_f:w.off_f + H] + w.f_bias) / w.cap))
    else:
        i, f = x.new_zeros(n, H), w.log_decay.expand(n, H)
    return (q * w.q_scale, k * w.k_scale, x[:, w.off_v:w.off_v + vd].reshape(n, H, w.vdim), i, f,
            x[:, w.off_g:w.off_g + vd])


def _portion_ref(proj, w: MemoryWeights, states, slot, pos0, out) -> None:
    """Consecutive tokens of one sequence from position ``pos0``; updates the slot's state."""
    n = proj.shape[0]
    q, k, v, i, f, g = _rows_ref(proj, w, torch.arange(pos0, pos0 + n, device=proj.device))
    state, nrm, top = states
    for t in (state, nrm, top):
        if t is not None and pos0 == 0:
            t[slot].zero_()
    S = state[slot]
    N, m = (nrm[slot, :, 0].clone(), top[slot, :, 0].clone()) if w.gated else (None, S.new_zeros(w.heads))
    for t in range(n):
        new = torch.maximum(f[t] + m, i[t])
        a, b = torch.exp(f[t] + m - new), torch.exp(i[t] - new)
        m = new
        S *= a[:, None, None]
        S += (b[:, None] * k[t])[:, :, None] * v[t][:, None, :]
        o = torch.matmul(q[t][:, None], S)[:, 0]
        if w.gated:
            N *= a[:, None]
            N += b[:, None] * k[t]
            o = o / (torch.maximum((N * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6)[:, None]
        o = (o / torch.sqrt(o.pow(2).mean(-1, keepdim=True) + w.eps)).flatten()
        if w.norm is not None:
            o = o * w.norm
        out[t] = (o * (F.silu(g[t]) if w.act == "silu" else torch.sigmoid(g[t]))).to(out.dtype)
    if w.gated:
        nrm[slot], top[slot] = N[:, None], m[:, None]


def _args(proj, w: MemoryWeights, states, out) -> dict:
    state, nrm, top = states
    H, n = w.heads, memory_slices(w.vdim)
    assert proj.dim() == 2 and proj.stride(1) == 1
    assert H * w.dim <= w.off_k and w.off_k + H * w.dim <= w.off_v
    assert max(w.off_v, w.off_g) + H * w.vdim <= proj.shape[1]
    assert state.dtype == torch.float32 and state.is_contiguous()
    assert state.shape[1:] == (H, w.dim, w.vdim) and 1 <= w.dim <= 256 and w.vdim <= 1024
    assert w.rot_dims == 0 or (w.rope.dtype == torch.float32 and w.rope.is_contiguous()
                               and w.rope.shape[1] == w.rot_dims <= w.dim and w.rot_dims % 2 == 0)
    small = (w.i_bias, w.f_bias) if w.gated else (w.log_decay,)
    for t in small:
        assert t.dtype == torch.float32 and t.numel() == H and t.is_contiguous()
    if w.gated:
        assert max(w.off_i, w.off_f) + H <= proj.shape[1] and w.cap > 0
        assert nrm.shape[1:] == (H, n, w.dim) and top.shape[1:] == (H, n)
        for t in (nrm, top):
            assert t.dtype == torch.float32 and t.is_contiguous() and t.shape[0] == state.shape[0]
    assert w.norm is None or (w.norm.dtype == torch.float32 and w.norm.numel() == H * w.vdim)
    assert out.shape[0] == proj.shape[0] and out.shape[1] >= H * w.vdim and out.stride(1) == 1
    assert out.dtype == proj.dtype
    return dict(proj=proj.data_ptr(), ldp=proj.stride(0), off_k=w.off_k, off_v=w.off_v,
                off_g=w.off_g, off_i=w.off_i, off_f=w.off_f, H=H, dim=w.dim, vdim=w.vdim,
                q_scale=float(w.q_scale), k_scale=float(w.k_scale), cos_sin=ptr(w.rope),
                rot_dims=w.rot_dims, log_decay=ptr(w.log_decay), i_bias=ptr(w.i_bias),
                f_bias=ptr(w.f_bias), cap=float(w.cap), norm_w=ptr(w.norm),
                silu=int(w.act == "silu"), eps=float(w.eps), state=state.data_ptr(), nrm=ptr(nrm),
                top=ptr(top), slices=n, out=out.data_ptr(), ldo=out.stride(0), nseg=0, rows=0)


def memory_scan(proj: torch.Tensor, w: MemoryWeights, states: tuple, p: Portions,
                out: torch.Tensor, portions: int | None = None, plain: bool = False) -> torch.Tensor:
    """The recurrence over packed portions (the first ``portions`` of them), each continuing its
    slot's state, with norm and gate of the read-out.  Leaves the state as of each portion's last
    token; rows in no portion are not written.  ``states``: (matrices [slots, heads, dim, vdim],
    and for the mLSTM normalisers [slots, heads, slices, dim], running maxima [slots, heads,
    slices]).
    ``plain``: token by token also where the chunk kernel takes the sizes."""
    n = p.seg_row.numel() if portions is None else portions
    if not on_gpu(proj):
        for s in range(n):
            slot, r0, ln, p0 = (int(t[s]) for t in (p.seg_state, p.seg_row, p.seg_len, p.seg_pos))
            if slot < 0:
                out[r0:r0 + ln] = 0
            else:
                _portion_ref(proj[r0:r0 + ln], w, states, slot, p0, out[r0:r0 + ln, :w.heads * w.vdim])
        return out
    if n == 0:
        return out
    a = _args(proj, w, states, out)
    for t in (p.seg_row, p.seg_len, p.seg_pos, p.seg_state):
        assert t.dtype == torch.int32 and t.is_cuda and t.numel() >= n
    a.update(seg_row=p.seg_row.data_ptr(), seg_len=p.seg_len.data_ptr(),
             seg_pos=p.seg_pos.data_ptr(), seg_state=p.seg_state.data_ptr(), nseg=n,
             rows=proj.shape[0])
    check(hipk().memory_scan(int(proj.dtype == torch.float32), a, int(plain), stream_ptr(proj)),
          "memory_scan")
    return out


def memory_decode(proj: torch.Tensor, w: MemoryWeights, states: tuple, positions: torch.Tensor,
                  row_state: torch.Tensor, out: torch.Tensor) -> torch.Tensor:
    """One token per sequence: rotation, gates, recurrence, norm and gate in one launch."""
    B = proj.shape[0]
    if not on_gpu(proj):
        for b in range(B):
            slot = int(row_state[b])
            if slot < 0:
                out[b] = 0
            else:
                _portion_ref(proj[b:b + 1], w, states, slot, int(positions[b]),
                             out[b:b + 1, :w.heads * w.vdim])
        return out
    a = _args(proj, w, states, out)
    assert positions.dtype == row_state.dtype == torch.int32
    assert positions.numel() >= B and row_state.numel() >= B
    a.update(positions=positions.data_ptr(), row_state=row_state.data_ptr(), rows=B)
    check(hipk().memory_decode(int(proj.dtype == torch.float32), a, stream_ptr(proj)),
          "memory_decode")
    return out
