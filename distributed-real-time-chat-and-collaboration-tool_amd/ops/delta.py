"""Gated delta rule with per-channel decay: short convolutions, recurrence, gated output norm.

HIP kernels: csrc/kernels/delta_rule.hip.  A sequence's state is a 32-bit matrix per head and a
ring of its last ``taps`` convolution inputs (entry = position % taps), both addressed by the
state slot its rows carry; slot -1 marks padding rows, position 0 starts from zero whatever
the slot held.
"""
from __future__ import annotations

from dataclasses import dataclass

import torch
import torch.nn.functional as F

from ._ext import check, hipk, on_gpu, stream_ptr


@dataclass
class DeltaWeights:
    """Small per-layer operands, 32-bit."""
    conv: torch.Tensor      # [taps, channels]: q | k | v channels
    a_exp: torch.Tensor     # [heads] exp(A_log)
    dt_bias: torch.Tensor   # [heads * dim]
    norm: torch.Tensor      # [vdim]
    eps: float
    heads: int
    kv_heads: int
    dim: int
    vdim: int

    @property
    def taps(self) -> int:
        return self.conv.shape[0]

    @property
    def channels(self) -> int:
        return self.conv.shape[1]


@dataclass
class Portions:
    """Packed rows by sequence, for the recurrent layers of a step."""
    seg_row: torch.Tensor    # int32 [n] first row
    seg_len: torch.Tensor
    seg_pos: torch.Tensor    # position of the first row
    seg_state: torch.Tensor  # state slot (-1: padding)
    row_off: torch.Tensor    # int32 [rows] rows of the same portion ahead of this one
    row_state: torch.Tensor  # int32 [rows]
    max_len: int


def _conv_row_ref(w: DeltaWeights, proj, ring, row, off, pos, slot):
    taps, C = w.conv.shape
    acc = torch.zeros(C, device=proj.device)
    for j in range(min(taps, pos + 1)):
        x = proj[row - j, :C] if j <= off else ring[slot, (pos - j) % taps]
        acc += x.float() * w.conv[taps - 1 - j]
    return F.silu(acc).to(proj.dtype)


def short_conv(proj: torch.Tensor, w: DeltaWeights, ring: torch.Tensor, positions: torch.Tensor,
               p: Portions) -> torch.Tensor:
    """Causal convolution + SiLU of the first ``channels`` columns of packed rows."""
    rows, C = p.row_state.numel(), w.channels
    out = torch.empty((rows, C), dtype=proj.dtype, device=proj.device)
    if not on_gpu(proj):
        for r in range(rows):
            slot = int(p.row_state[r])
            out[r] = _conv_row_ref(w, proj, ring, r, int(p.row_off[r]), int(positions[r]), slot) \
                if slot >= 0 else 0
        return out
    _check_weights(proj, w, ring)
    assert proj.shape[0] >= rows and positions.dtype == torch.int32 and positions.numel() >= rows
    assert p.row_off.dtype == p.row_state.dtype == torch.int32 and p.row_off.numel() == rows
    check(hipk().short_conv(int(proj.dtype == torch.float32), out.data_ptr(), proj.data_ptr(),
                            proj.stride(0), w.conv.data_ptr(), ring.data_ptr(),
                            positions.data_ptr(), p.row_off.data_ptr(), p.row_state.data_ptr(),
                            rows, C, w.taps, stream_ptr(proj)), "short_conv")
    return out


def _check_weights(proj, w: DeltaWeights, ring) -> None:
    assert proj.dim() == 2 and proj.stride(1) == 1 and proj.shape[1] >= w.channels
    assert w.channels == 2 * w.kv_heads * w.dim + w.heads * w.vdim
    assert w.heads % w.kv_heads == 0 and w.dim <= 256 and w.vdim <= 512
    assert ring.is_contiguous() and ring.shape[1:] == (w.taps, w.channels)
    assert ring.dtype == proj.dtype
    for t, n in ((w.a_exp, w.heads), (w.dt_bias, w.heads * w.dim), (w.norm, w.vdim)):
        assert t.dtype == torch.float32 and t.numel() == n and t.is_contiguous()
    assert w.conv.dtype == torch.float32 and w.conv.is_contiguous()


def _args(proj, off_b, w: DeltaWeights, ring, state, decay, gate, out) -> dict:
    _check_weights(proj, w, ring)
    assert state.dtype == torch.float32 and state.is_contiguous()
    assert state.shape[1:] == (w.heads, w.dim, w.vdim)
    assert decay.stride(1) == 1 and decay.shape[1] >= w.heads * w.dim
    assert gate.stride(1) == 1 and gate.shape[1] >= w.heads * w.vdim
    assert decay.dtype == gate.dtype == proj.dtype and off_b + w.heads <= proj.shape[1]
    return dict(proj=proj.data_ptr(), ldp=proj.stride(0), off_b=off_b, conv_w=w.conv.data_ptr(),
                ring=ring.data_ptr(), state=state.data_ptr(), decay=decay.data_ptr(),
                ld_decay=decay.stride(0), gate=gate.data_ptr(), ld_gate=gate.stride(0),
                a_exp=w.a_exp.data_ptr(), dt_bias=w.dt_bias.data_ptr(),
                norm_w=w.norm.data_ptr(), eps=float(w.eps), H=w.heads, Hk=w.kv_heads, dim=w.dim,
                vdim=w.vdim, taps=w.taps, C=w.channels, out=out.data_ptr(), nseg=0, rows=0)


def _token_ref(w: DeltaWeights, x, beta_in, decay, gate, S):
    """One token from its convolved channels; updates S [heads, dim, vdim] in place."""
    kd = w.kv_heads * w.dim
    q = x[:kd].float().view(w.kv_heads, w.dim)
    k = x[kd:2 * kd].float().view(w.kv_heads, w.dim)
    v = x[2 * kd:].float().view(w.heads, w.vdim)
    grp = w.heads // w.kv_heads
    q = (q * torch.rsqrt(q.pow(2).sum(-1, keepdim=True) + 1e-6) * w.dim ** -0.5).repeat_interleave(grp, 0)
    k = (k * torch.rsqrt(k.pow(2).sum(-1, keepdim=True) + 1e-6)).repeat_interleave(grp, 0)
    g = torch.exp(-w.a_exp[:, None] * F.softplus(decay.float() + w.dt_bias).view(w.heads, w.dim))
    S *= g[:, :, None]
    u = torch.sigmoid(beta_in.float())[:, None] * (v - torch.matmul(k[:, None], S)[:, 0])
    S += k[:, :, None] * u[:, None, :]
    o = torch.matmul(q[:, None], S)[:, 0]
    o = o * torch.rsqrt(o.pow(2).mean(-1, keepdim=True) + w.eps) * w.norm
    return (o * torch.sigmoid(gate.float()).view(w.heads, w.vdim)).flatten()


def delta_scan(proj: torch.Tensor, off_b: int, conv: torch.Tensor, w: DeltaWeights,
               ring: torch.Tensor, state: torch.Tensor, decay: torch.Tensor, gate: torch.Tensor,
               p: Portions, columns: int = 0) -> torch.Tensor:
    """The recurrence over packed portions, each continuing its slot's state (from zero at
    position 0), then output norm and gate -> [rows, heads * vdim].  Leaves the state and the
    ring as of each portion's last token.  Rows in no portion are not written.  ``columns`` 0:
    chunks of 8 tokens on the fp32 MFMA where the sizes allow it; 2 / 4: token by token, with
    that many state columns to a lane."""
    rows = p.row_state.numel()
    out = torch.empty((rows, w.heads * w.vdim), dtype=proj.dtype, device=proj.device)
    if not on_gpu(proj):
        out.zero_()
        for s in range(p.seg_row.numel()):
            slot, r0, n, p0 = (int(t[s]) for t in (p.seg_state, p.seg_row, p.seg_len, p.seg_pos))
            if slot < 0:
                continue
            S = state[slot]
            if p0 == 0:
                S.zero_()
            for r in range(r0, r0 + n):
                out[r] = _token_ref(w, conv[r], proj[r, off_b:off_b + w.heads], decay[r], gate[r],
                                    S).to(out.dtype)
            for t in range(max(0, n - w.taps), n):
                ring[slot, (p0 + t) % w.taps] = proj[r0 + t, :w.channels]
        return out
    a = _args(proj, off_b, w, ring, state, decay, gate, out)
    n = p.seg_row.numel()
    for t in (p.seg_row, p.seg_len, p.seg_pos, p.seg_state):
        assert t.dtype == torch.int32 and t.is_cuda and t.numel() == n
    assert conv.is_contiguous() and conv.shape[1] == w.channels and conv.dtype == proj.dtype
    a.update(conv=conv.data_ptr(), seg_row=p.seg_row.data_ptr(), seg_len=p.seg_len.data_ptr(),
             seg_pos=p.seg_pos.data_ptr(), seg_state=p.seg_state.data_ptr(), nseg=n)
    check(hipk().delta_scan(int(proj.dtype == torch.float32), a,
                            columns, stream_ptr(proj)), "delta_scan")
    return out


def delta_decode(proj: torch.Tensor, off_b: int, w: DeltaWeights, ring: torch.Tensor,
                 state: torch.Tensor, decay: torch.Tensor, gate: torch.Tensor,
                 positions: torch.Tensor, row_state: torch.Tensor) -> torch.Tensor:
    """One token per sequence: convolution, recurrence, output norm and gate in one launch."""
    B = proj.shape[0]
    out = torch.empty((B, w.heads * w.vdim), dtype=proj.dtype, device=proj.device)
    if not on_gpu(proj):
        for b in range(B):
            slot, pos = int(row_state[b]), int(positions[b])
            if slot < 0:
                out[b] = 0
                continue
            x = _conv_row_ref(w, proj, ring, b, 0, pos, slot)
            if pos == 0:
                state[slot].zero_()
            out[b] = _token_ref(w, x, proj[b, off_b:off_b + w.heads], decay[b], gate[b],
                                state[slot]).to(out.dtype)
            ring[slot, pos % w.taps] = proj[b, :w.channels]
        return out
    a = _args(proj, off_b, w, ring, state, decay, gate, out)
    assert positions.dtype == row_state.dtype == torch.int32
    assert positions.numel() >= B and row_state.numel() >= B
    a.update(positions=positions.data_ptr(), row_state=row_state.data_ptr(), rows=B)
    check(hipk().delta_decode(int(proj.dtype == torch.float32), a, stream_ptr(proj)),
          "delta_decode")
    return out
