"""Fused mixture-of-experts layer (router top-k -> grouped expert GEMMs -> combine).

HIP kernels: csrc/kernels/moe.hip.  One call enqueues four kernels with
static launch shapes (the per-expert tile table lives on the device), so the
layer is hipGraph-capturable and the Mixtral decode step replays with no
host synchronisation and exact sparse FLOPs (the earlier graph path ran every
expert on every token).  SURVEY.md §2 K8.

Routing semantics: top-k of the router logits, softmax over the selected k logits (as much as a
softmax over all experts divided by the chosen ones' sum); ties pick the lower expert id.  With
``groups`` the experts form equal groups of neighbours and a token chooses within its ``keep``
groups of the largest logits.  With expert parallelism a
rank holds experts [e_off, e_off + e_local) and returns only their
contribution (the caller all-reduces over the EP group).
"""
from __future__ import annotations

import os

import torch
import torch.nn.functional as F

from ._ext import check, hipk, on_gpu, stream_ptr
from .activation import ACTS, act_glu_ref

# Largest token chunk per kernel call: bounds the workspace (P = chunk * k rows of [I] and [H]
# intermediates: ~3 GB for Mixtral).  One Mixtral prefill step (ModelConfig.prefill_chunk,
# 32k tokens) in one call: 8k rows per expert on variant 4 (profiles/r6j: the 16k-token layer
# 8.94 ms in one call vs 9.56 ms in two of 8192; profiles/r6t: the batch-1024 wave +1.6 % with
# 32k-token prefill steps and MoE calls).
MOE_CHUNK = int(os.environ.get("DRTC_MOE_CHUNK", "32768"))

MAX_TOP_K, MAX_GROUPS = 16, 64  # of the routing kernel

# Grouped-GEMM structure (csrc/kernels/moe.hip): 0 = 128-row two-barrier,
# 1 = 128-row 3-stage pipeline, 2 = 256-row 3-stage pipeline, 3 = gemm_xd's grouped mode
# (csrc/kernels/gemm_xd.hip: XCD-partitioned tiles, GLU epilogue, split-K, non-temporal
# weights where an expert's rows fit one tile), 4 = token rows gathered into expert order, then
# gemm_w4's grouped persistent 256 x 256 form (csrc/kernels/gemm_w4.hip; prefill-sized rows per
# expert), -1 = by rows per expert (4 from 256 rows per expert, 3 from 96).
MOE_GEMM_VARIANT = int(os.environ.get("DRTC_MOE_VARIANT", "-1"))
# gemm_xd forms of variant 3 (mt * 100 + nf * 10 + splitk, + 1000 non-temporal; 0 = by rows
# per expert, csrc/kernels/moe.hip launch_moe)
MOE_GU_FORM = int(os.environ.get("DRTC_MOE_GU_FORM", "0"))
MOE_DN_FORM = int(os.environ.get("DRTC_MOE_DN_FORM", "0"))


def route_ref(router_logits: torch.Tensor, top_k: int, groups: int = 1, keep: int = 1):
    """(expert ids [T, k], weights [T, k] fp32) with the kernel's tie rule."""
    lg = router_logits.float()
    if groups > 1:
        best = lg.view(lg.shape[0], groups, -1).amax(-1)
        order = torch.sort(best, dim=-1, descending=True, stable=True).indices
        closed = torch.ones_like(best, dtype=torch.bool).scatter_(1, order[:, :keep], False)
        lg = lg.masked_fill(closed.repeat_interleave(lg.shape[1] // groups, 1), float("-inf"))
    v, i = torch.sort(lg, dim=-1, descending=True, stable=True)
    return i[:, :top_k], torch.softmax(v[:, :top_k], dim=-1)


def fused_moe_ref(x: torch.Tensor, router_logits: torch.Tensor, w_gu: torch.Tensor,
                  w_dn: torch.Tensor, top_k: int, act: str = "silu", e_off: int = 0,
                  groups: int = 1, keep: int = 1, limit: float = 0.0, stream: torch.Tensor | None = None,
                  y: torch.Tensor | None = None) -> torch.Tensor:
    """fp32-accumulated PyTorch reference of :func:`fused_moe`."""
    topi, wts = route_ref(router_logits, top_k, groups, keep)
    out = torch.zeros(x.shape[0], x.shape[1], dtype=torch.float32, device=x.device)
    for le in range(w_gu.shape[0]):
        tok, slot = torch.nonzero(topi == e_off + le, as_tuple=True)
        if tok.numel() == 0:
            continue
        xe = x.index_select(0, tok).float()
        h = xe @ w_gu[le].float().t()
        h = h.relu().square() if act == "relu2" else act_glu_ref(h, act, limit)
        h = h.to(x.dtype).float()
        ye = (h @ w_dn[le].float().t()).to(x.dtype).float()
        out.index_add_(0, tok, ye * wts[tok, slot].unsqueeze(1))
    if stream is not None:
        stream += out[:, :stream.shape[1]] + y.float()
        return stream.to(x.dtype)
    return out.to(x.dtype)


def workspace_bytes(tokens: int, hidden: int, inter: int, e_local: int, top_k: int,
                    f32: bool = False) -> int:
    return int(hipk().moe_workspace_bytes(tokens, hidden, inter, e_local, top_k, int(f32)))


def make_workspace(tokens: int, hidden: int, inter: int, e_local: int, top_k: int,
                   device, f32: bool = False) -> torch.Tensor:
    """Persistent scratch for up to ``tokens`` tokens per call (allocate once,
    before any graph capture; also creates the device's split-K GEMM workspace that the
    gemm_xd forms of variant 3 use)."""
    from .gemm import gemm_workspace

    n = workspace_bytes(min(tokens, MOE_CHUNK), hidden, inter, e_local, top_k, f32)
    if torch.device(device).type == "cuda":
        gemm_workspace(torch.device(device))
    return torch.empty(n, dtype=torch.uint8, device=device)


# fused_moe reads the router GEMM's [E, T] output in place (DRTC_ROUTER_VIEW=0: the
# transposed copy of round 5's first router form, for A/B)
ROUTER_VIEW = os.environ.get("DRTC_ROUTER_VIEW", "1") != "0"


def router_logits(x: torch.Tensor, w_router: torch.Tensor, contiguous: bool = True) -> torch.Tensor:
    """Router logits x [T, H] . w_router [E, H]^T -> [T, E], on the skinny HIP GEMM
    transposed: the E router rows are the kernel's few activation rows and the T tokens its
    streamed weight rows, so x is read once and no library GEMM runs in the MoE layer (ref
    llm_server/llm_server.py:403: the suggestions model).  ``contiguous=False`` returns the
    kernel's [E, T] output as a transposed [T, E] view (strides (1, T)), which ``fused_moe``
    reads in place (no transpose copy per layer).  A T that is not a multiple of the kernel's
    16-row block is zero-padded up to one, so every batch size routes through the same kernel
    and the same rounding (top-k choices on near-tied logits do not depend on T); E > 8 goes
    to F.linear."""
    from . import gemm as G

    T, H = x.shape
    E = w_router.shape[0]
    Tp = -(-T // 16) * 16
    if (on_gpu(x) and x.is_contiguous() and w_router.is_contiguous() and E <= 8 and T > 0
            and G.skinny_supports(3, E, Tp, H, w_router.stride(0))):
        if Tp != T:
            xp = x.new_zeros((Tp, H))
            xp[:T].copy_(x)
            x = xp
        y = G.skinny_linear(w_router, x, variant=3).t()[:T]
        return y.contiguous() if contiguous or not ROUTER_VIEW else y
    return F.linear(x, w_router)


def router_logits_f32(x: torch.Tensor, w_router: torch.Tensor) -> torch.Tensor:
    """Router logits x [T, H] . w_router [E, H]^T in fp32, [T, E] (for bf16 operands the transposed
    view of an [E, T] tensor).  Every token's sum runs in the same order whatever the batch."""
    if not on_gpu(x):
        return F.linear(x.float(), w_router.float())
    T, H = x.shape
    E = w_router.shape[0]
    if x.dtype == torch.float32:
        return F.linear(x, w_router)
    assert x.dtype == w_router.dtype == torch.bfloat16 and w_router.is_contiguous()
    assert x.stride(1) == 1 and x.stride(0) % 8 == 0 and H % 8 == 0 and E <= 256
    out = torch.empty((E, T), dtype=torch.float32, device=x.device)
    check(hipk().moe_router(out.data_ptr(), x.data_ptr(), x.stride(0), w_router.data_ptr(), T, E, H,
                            stream_ptr(x)), "moe_router")
    return out.t()


def fused_moe(x: torch.Tensor, router_logits: torch.Tensor, w_gu: torch.Tensor,
              w_dn: torch.Tensor, top_k: int, act: str = "silu", num_experts: int | None = None,
              e_off: int = 0, workspace: torch.Tensor | None = None,
              out: torch.Tensor | None = None, variant: int | None = None,
              gu_form: int | None = None, dn_form: int | None = None, groups: int = 1,
              keep: int = 1, limit: float = 0.0, stream: torch.Tensor | None = None,
              y: torch.Tensor | None = None) -> torch.Tensor:
    """y[t] = sum_j w[t,j] * down_e(act(gate_e x_t) * up_e x_t) over the top-k experts; act
    "relu2": down_e(relu(up_e x_t)^2), w_gu [E_local, I, H].

    ``stream`` [T, W <= H] fp32: the result is added to it together with ``y`` [T, W], and the
    stream is returned in x's type (itself in fp32).

    x [T, H] bf16 (H % 128 == 0, I % 64 == 0) or fp32 (any size); router_logits [T, E] bf16 or
    fp32, row-major or the transposed view of an [E, T] tensor (``router_logits(...,
    contiguous=False)``); w_gu [E_local, 2I, H] ([gate | up] rows); w_dn [E_local, H, I] ("relu2"
    in bf16: I % 128 == 0).
    ``groups`` / ``keep``: group-limited choice; ``limit``: bound of the clamped activation.
    """
    if not on_gpu(x):
        r = fused_moe_ref(x, router_logits, w_gu, w_dn, top_k, act, e_off, groups, keep, limit,
                          stream, y)
        if out is not None:
            out.copy_(r)
            return out
        return r
    T, H = x.shape
    # every token count takes the fused kernels (prefill included: no host sync per layer;
    # the round-4 per-expert hipBLASLt path for T >= 4096 measured slower at T = 8192,
    # 6.05 / 5.86 ms fused vs 6.25 / 5.95 ms, profiles/r4ah, r4ak)
    E = num_experts if num_experts is not None else router_logits.shape[1]
    e_local, n_in, h2 = w_gu.shape
    inter = n_in if act == "relu2" else n_in // 2
    f32 = x.dtype == torch.float32
    assert x.dtype == w_gu.dtype == w_dn.dtype and x.is_contiguous()
    assert f32 or x.dtype == torch.bfloat16
    assert router_logits.dtype in (torch.bfloat16, torch.float32)
    assert router_logits.shape == (T, E) and h2 == H
    lts, les = router_logits.stride()
    assert (lts, les) == (E, 1) or (lts == 1 and les >= T), router_logits.stride()
    assert w_gu.is_contiguous() and w_dn.is_contiguous() and w_dn.shape == (e_local, H, inter)
    assert E <= 256 and 1 <= top_k <= min(MAX_TOP_K, E)
    assert f32 or (H % 128 == 0 and inter % (128 if act == "relu2" else 64) == 0)
    assert 1 <= groups <= MAX_GROUPS and E % groups == 0 and 1 <= keep <= groups
    assert top_k <= keep * (E // groups)
    W = H
    if stream is not None:
        W = stream.shape[1]
        assert stream.shape == y.shape == (T, W) and W <= H and stream.is_contiguous()
        assert stream.dtype == torch.float32 and y.dtype == x.dtype and y.stride(1) == 1
        assert out is None and (e_off, e_local) == (0, E)
        out = stream if f32 else x.new_empty(T, W)
    elif out is None:
        out = torch.empty_like(x)
    assert out.is_contiguous() and out.shape == (T, W)
    chunk = min(T, MOE_CHUNK) if T else 1
    need = workspace_bytes(chunk, H, inter, e_local, top_k, f32)
    if workspace is None or workspace.numel() < need:
        assert not torch.cuda.is_current_stream_capturing(), \
            "fused_moe under graph capture needs a preallocated workspace"
        workspace = torch.empty(need, dtype=torch.uint8, device=x.device)
    lib, st = hipk(), stream_ptr(x)
    # the split-K slabs / counters of the gemm_xd forms: the device's shared GEMM workspace
    # (same stream), only when it exists already (never created inside a graph capture)
    from . import gemm as _gemm

    key = x.device.index if x.device.index is not None else torch.cuda.current_device()
    gws = _gemm._ws.get(key)
    slab, cnt = gws if gws is not None else (None, None)
    for t0 in range(0, T, MOE_CHUNK):
        n = min(MOE_CHUNK, T - t0)
        check(lib.moe(out[t0].data_ptr(), x[t0].data_ptr(), router_logits[t0].data_ptr(),
                      w_gu.data_ptr(), w_dn.data_ptr(), n, H, inter, E, top_k, e_off, e_local,
                      ACTS[act], workspace.data_ptr(), workspace.numel(),
                      MOE_GEMM_VARIANT if variant is None else variant,
                      MOE_GU_FORM if gu_form is None else gu_form,
                      MOE_DN_FORM if dn_form is None else dn_form,
                      slab.data_ptr() if slab is not None else 0,
                      slab.numel() * 4 if slab is not None else 0,
                      cnt.data_ptr() if cnt is not None else 0,
                      cnt.numel() if cnt is not None else 0, lts, les, int(f32),
                      int(router_logits.dtype == torch.float32), groups, keep, float(limit),
                      0 if stream is None else stream[t0].data_ptr(),
                      0 if stream is None else y[t0].data_ptr(),
                      0 if stream is None else y.stride(0), W, st), "moe")
    return out

