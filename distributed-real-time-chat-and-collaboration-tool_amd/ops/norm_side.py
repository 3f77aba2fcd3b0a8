"""The residual stream of joint layers: layer norm without bias behind an embedding lookup or the
add of a token's side input (itself RMS-normed), the add of both sublayers, and the side input's
gate.

HIP kernels: csrc/kernels/norm_side.hip.
"""
from __future__ import annotations

import math

import torch

from ._ext import check, hipk, on_gpu, ptr, stream_ptr


def side_norm(h: torch.Tensor, w: torch.Tensor, eps: float, y: torch.Tensor | None = None,
              y_norm: torch.Tensor | None = None, ids: torch.Tensor | None = None,
              embed: torch.Tensor | None = None, embed_scale: float = 1.0,
              width: int | None = None, dtype=torch.bfloat16) -> torch.Tensor:
    """Layer norm (weight w, no bias) of the 32-bit residual stream h [rows, W], after
    h += y / sqrt(mean(y^2) + eps) * y_norm or h = embed_scale * embed[ids]; h is updated in
    place.  w, y_norm: float32.  ``width`` > W: zeros behind the first W output columns."""
    rows, W = h.shape
    N = width or W
    if not on_gpu(h):
        if ids is not None:
            h.copy_(embed[ids.long()].float() * embed_scale)
        elif y is not None:
            yf = y.float()
            h += yf / torch.sqrt(yf.pow(2).mean(-1, keepdim=True) + eps) * y_norm
        d = h - h.mean(-1, keepdim=True)
        n = d / torch.sqrt(d.pow(2).mean(-1, keepdim=True) + eps) * w
        return torch.nn.functional.pad(n, (0, N - W)).to(dtype)
    assert h.dtype == w.dtype == torch.float32 and h.is_contiguous() and w.is_contiguous()
    assert w.numel() == W and N >= W and W <= 16384
    assert y is None or (y.shape == (rows, W) and y.stride(1) == 1 and y.dtype == dtype
                         and y_norm.dtype == torch.float32 and y_norm.numel() == W
                         and y_norm.is_contiguous())
    assert ids is None or (ids.dtype == torch.int32 and ids.numel() == rows and ids.is_contiguous()
                           and embed.is_contiguous() and embed.dtype == dtype
                           and embed.shape[1] == W)
    out = torch.empty((rows, N), dtype=dtype, device=h.device)
    check(hipk().side_norm(int(dtype == torch.float32), dict(
        out=out.data_ptr(), ldo=N, h=h.data_ptr(), y=ptr(y), ldy=y.stride(0) if y is not None else 0,
        yw=ptr(y_norm), ids=ptr(ids), embed=ptr(embed), embed_scale=float(embed_scale),
        w=w.data_ptr(), W=W, eps=float(eps), rows=rows), stream_ptr(h)), "side_norm")
    return out


def stream_add(h: torch.Tensor, y: torch.Tensor) -> torch.Tensor:
    """h += y on the 32-bit stream; the stream in y's type (h itself in fp32)."""
    if not on_gpu(h):
        h += y.float()
        return h.to(y.dtype)
    rows, W = h.shape
    assert h.dtype == torch.float32 and h.is_contiguous()
    assert y.shape == (rows, W) and y.stride(1) == 1
    out = h if y.dtype == torch.float32 else torch.empty_like(h, dtype=y.dtype)
    check(hipk().stream_add(int(y.dtype == torch.float32), out.data_ptr(), h.data_ptr(),
                            y.data_ptr(), y.stride(0), rows, W, stream_ptr(h)), "stream_add")
    return out


SIDE_GEMM_ROWS = 512  # larger steps form z in a GEMM of its own


def side_input(x: torch.Tensor, w: torch.Tensor, embed: torch.Tensor, ids: torch.Tensor,
               layer: int) -> torch.Tensor:
    """gelu_tanh(x @ w.T) times the tokens' own inputs to ``layer``: w [dim, W], embed [vocab,
    layers * dim]; one kernel for decode-sized batches in bf16."""
    from .gemm import linear

    rows, K = x.shape
    dim = w.shape[0]
    if not (on_gpu(x) and x.dtype == torch.bfloat16 and rows <= SIDE_GEMM_ROWS and K % 8 == 0):
        return side_gate(linear(x, w), embed, ids, layer)
    assert x.is_contiguous() and w.is_contiguous() and embed.is_contiguous()
    assert x.dtype == w.dtype == embed.dtype and w.shape[1] == K
    assert ids.dtype == torch.int32 and ids.numel() == rows and ids.is_contiguous()
    assert (layer + 1) * dim <= embed.shape[1]
    out = x.new_empty(rows, dim)
    check(hipk().side_gate_gemm(out.data_ptr(), x.data_ptr(), w.data_ptr(), embed.data_ptr(),
                                embed.shape[1], layer * dim, ids.data_ptr(), rows, dim, K,
                                stream_ptr(x)), "side_gate_gemm")
    return out


def side_gate(z: torch.Tensor, embed: torch.Tensor, ids: torch.Tensor, layer: int) -> torch.Tensor:
    """gelu_tanh(z) times the tokens' own inputs to ``layer``: embed [vocab, layers * dim],
    z [rows, dim]."""
    rows, dim = z.shape
    if not on_gpu(z):
        e = embed[ids.long(), layer * dim:(layer + 1) * dim].float()
        x = z.float()
        return (0.5 * x * (1 + torch.tanh(math.sqrt(2 / math.pi) * (x + 0.044715 * x.pow(3)))) * e).to(z.dtype)
    assert z.is_contiguous() and embed.is_contiguous() and embed.dtype == z.dtype
    assert ids.dtype == torch.int32 and ids.numel() == rows and ids.is_contiguous()
    assert (layer + 1) * dim <= embed.shape[1]
    out = torch.empty_like(z)
    check(hipk().side_gate(int(z.dtype == torch.float32), out.data_ptr(), z.data_ptr(),
                           embed.data_ptr(), embed.shape[1], layer * dim, ids.data_ptr(), rows, dim,
                           stream_ptr(z)), "side_gate")
    return out
