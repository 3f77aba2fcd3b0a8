"""Paged KV cache sized for MI355X HBM (288 GB per GPU).

One contiguous allocation per engine, carved into per-layer views:
  k[layer] : [num_blocks, Hkv, 32, D]   token-major (MFMA A-operand rows)
  v[layer] : [num_blocks, Hkv, D, 32]   storage shape; a block holds 8 groups
             of 4 tokens, dim-major inside a group (P.V A-operand: 4 tokens of
             one dim = 8 contiguous bytes; a decode write spans 2*D bytes)
The block count is derived from the free HBM left after the weights
(``torch.cuda.mem_get_info``) times ``kv_fraction``; on a 288 GB MI355X with
Llama-3-8B that is ~1.5 M cached tokens.  Blocks are handed out by the
native :class:`BlockAllocator` (C++ free list, see csrc/runtime).  No
reference counterpart: the reference keeps no model state (hosted Gemini,
llm_server/llm_server.py:33).
"""
from __future__ import annotations

import torch

from ..ops import KV_BLOCK, latent_width, memory_slices, pad8, talk_cache_shapes
from ..models.config import (GatedAverage, GroupedAttention, HybridConfig, Layer, LatentAttention,
                             MatrixMemory, ModelConfig, Retention, TalkingAttention)
from .block_allocator import BlockAllocator


def blocks_for_budget(cfg: ModelConfig, hkv_local: int, n_layers: int, budget_bytes: int,
                      dtype_bytes: int = 2) -> int:
    per_block = 2 * n_layers * hkv_local * KV_BLOCK * cfg.head_dim * dtype_bytes
    return max(0, budget_bytes // per_block)


class PagedKVCache:
    def __init__(self, cfg: ModelConfig, hkv_local: int, num_blocks: int,
                 device: torch.device | str, dtype=torch.bfloat16):
        self.cfg = cfg
        self.block_size = KV_BLOCK
        self.num_blocks = int(num_blocks)
        self.hkv = hkv_local
        D = cfg.head_dim
        L = cfg.num_layers
        per = self.num_blocks * hkv_local * KV_BLOCK * D
        # zero-filled: stale/uninitialised bytes in partially filled blocks
        # must never be NaN (they are multiplied by p = 0 in P.V).
        self.buffer = torch.zeros((L, 2, per), dtype=dtype, device=device)
        self.layers = []
        for l in range(L):
            k = self.buffer[l, 0].view(self.num_blocks, hkv_local, KV_BLOCK, D)
            v = self.buffer[l, 1].view(self.num_blocks, hkv_local, D, KV_BLOCK)
            self.layers.append((k, v))
        # block 0 is reserved as the padding target of graph-padded slots
        self.allocator = BlockAllocator(self.num_blocks, reserved=1)
        self.states = None  # no recurrent state

    def __getitem__(self, i):
        return self.layers[i]

    def __len__(self):
        return len(self.layers)

    @property
    def bytes(self) -> int:
        return self.buffer.numel() * self.buffer.element_size()

    @property
    def capacity_tokens(self) -> int:
        return (self.num_blocks - 1) * KV_BLOCK

    @staticmethod
    def auto_num_blocks(cfg: ModelConfig, hkv_local: int, device, kv_fraction: float = 0.85,
                        reserve_bytes: int = 8 << 30, max_blocks: int | None = None,
                        hbm_budget: float | None = None, weight_bytes: int | None = None,
                        min_blocks: int = 0) -> int:
        """KV blocks for an engine on ``device``: ``kv_fraction`` of the HBM free beyond
        ``reserve_bytes`` (activations, GEMM workspaces, graphs) - or, with ``hbm_budget``
        (engine groups sharing a GPU, llm.server --serve ...:mem=F), what is left of
        hbm_budget x the GPU's total HBM after the group's weights (``weight_bytes``; this
        process's allocations when not given) and the reserve, whatever the other groups on the
        GPU - in other processes or in this one - hold or start in what order."""
        per_block = 2 * cfg.num_layers * hkv_local * KV_BLOCK * cfg.head_dim * 2
        return _budget_blocks(cfg.name, per_block, 0, device, kv_fraction, reserve_bytes,
                              max_blocks, hbm_budget, weight_bytes, min_blocks)


def _budget_blocks(name: str, per_block: int, fixed: int, device, kv_fraction: float,
                   reserve_bytes: int, max_blocks: int | None, hbm_budget: float | None,
                   weight_bytes: int | None, min_blocks: int) -> int:
    """Blocks of ``per_block`` bytes beside ``fixed`` bytes of other cache (see
    PagedKVCache.auto_num_blocks)."""
    dev = torch.device(device)
    if dev.type == "cuda":
        # blocks the caching allocator holds but no tensor uses are free HBM here: release
        # them so that neither the free figure nor this process's own share counts them
        torch.cuda.empty_cache()
        free, total = torch.cuda.mem_get_info(dev)
        budget = int(max(0, free - reserve_bytes) * kv_fraction)
        if hbm_budget is not None:
            mine = torch.cuda.memory_reserved(dev) if weight_bytes is None else weight_bytes
            left = int(hbm_budget * total) - mine - reserve_bytes
            if max(left - fixed, 0) // max(1, per_block) < min_blocks:
                # ``min_blocks``: the cache of one max_model_len sequence
                raise ValueError(
                    f"{name}: an HBM budget of {hbm_budget:.2f} x {total / 1e9:.0f} GB "
                    f"on {dev} leaves {left / 1e9:.1f} GB for the KV cache after "
                    f"{mine / 1e9:.1f} GB of weights and the {reserve_bytes / 1e9:.0f} GB "
                    f"reserve: less than one {min_blocks}-block sequence needs")
            budget = min(budget, max(left, 0))
    else:
        budget = 256 << 20
    n = max(0, budget - fixed) // max(1, per_block)
    if max_blocks is not None:
        n = min(n, max_blocks)
    return max(n, 2)


def _layer_parts(l: Layer, dtype) -> tuple[list, list]:
    """What a layer's mixer caches: (shape, dtype) of its tensors per cache block, and per
    state slot."""
    m, f32 = l.mixer, torch.float32
    if isinstance(m, LatentAttention):
        if m.kv_from is not None:  # nothing of its own
            return [], []
        return [((KV_BLOCK, latent_width(m.kv_rank, m.rot_dim)), dtype)], []
    if isinstance(m, Retention):
        return [], [((m.heads, m.dim, m.vdim), f32)]
    if isinstance(m, MatrixMemory):
        n = memory_slices(m.vdim)
        return [], [((m.heads, m.dim, m.vdim), f32), ((m.heads, n, m.dim), f32), ((m.heads, n), f32)]
    if isinstance(m, TalkingAttention):
        return [(s, dtype) for s in talk_cache_shapes(m.kv_heads, m.dim, m.vdim)], []
    if isinstance(m, GroupedAttention):
        C = (m.heads + m.kv_heads) * pad8(m.dim) + m.kv_heads * pad8(m.vdim)
        return ([(s, dtype) for s in talk_cache_shapes(m.kv_heads, m.dim, m.vdim)],
                [((max(m.conv, 1) - 1, C), dtype)])
    if isinstance(m, GatedAverage):
        return [], [((pad8(m.width),), f32)]
    return [], [((m.conv, m.channels), dtype), ((m.heads, m.dim, m.vdim), f32)]


def _ring_part(cfg: HybridConfig, l: Layer) -> tuple | None:
    """Shape per state slot of a layer's ring of convolved sublayer inputs."""
    return (2 if l.ff else 1, cfg.conv_taps - 1, cfg.hidden_size) if cfg.conv_taps > 1 else None


def _plane_heads(cfg: HybridConfig) -> int:
    """Heads of the plane of scores that talking-heads layers share."""
    return max((l.mixer.heads for l in cfg.layers if isinstance(l.mixer, TalkingAttention)), default=0)


class HybridCache:
    """Cache of a model with mixed layer kinds: paged tokens for its attention layers, and
    state slots - one per live sequence - for its recurrent layers and convolved inputs.

      latent layer    [num_blocks, 32, latent_width]                      (ops/latent.py)
                      a layer with kv_from: the very tensor of the layer it reads
      talking layer   keys, values [num_blocks, ...]                      (ops/talking.py)
                      and the plane [num_blocks, heads, 32] of scores all such layers share
      grouped layer   keys, values as a talking layer's; ring [slots, taps - 1, channels] of
                      projected rows                                      (ops/grouped.py)
      delta layer     ring  [slots, taps, channels]       last convolution inputs
                      state [slots, heads, dim, vdim]     fp32
      average layer   state [slots, channels]             fp32
      retention layer state [slots, heads, dim, vdim]     fp32            (ops/memory.py)
      memory layer    state as a retention layer's; normaliser [slots, heads, slices, dim] and
                      running maximum [slots, heads, slices] of each column slice    fp32
      rings           [slots, sublayers, taps - 1, W]     convolved inputs, per layer

    Blocks come from ``allocator`` (block 0 is the padding target), slots from ``states``.
    A slot needs no clearing: a sequence starts from zero at its position 0 whatever the slot
    holds."""

    def __init__(self, cfg: HybridConfig, num_blocks: int, num_slots: int,
                 device: torch.device | str, dtype=torch.bfloat16):
        self.cfg, self.block_size = cfg, KV_BLOCK
        self.num_blocks, self.num_slots = int(num_blocks), int(num_slots)
        # zero-filled: rows behind a sequence's end are read (and masked) with its block

        def new(n, shape, dt):
            return torch.zeros((n, *shape), dtype=dt, device=device)

        heads = _plane_heads(cfg)
        self.plane = new(self.num_blocks, (heads, KV_BLOCK), torch.float32) if heads else None
        self.layers, self.rings = [], []
        for l in cfg.layers:
            block, slot = _layer_parts(l, dtype)
            ts = [new(self.num_blocks, *p) for p in block] + [new(self.num_slots, *p) for p in slot]
            if isinstance(l.mixer, TalkingAttention):
                ts.append(self.plane)
            j = getattr(l.mixer, "kv_from", None)
            self.layers.append(self.layers[j] if j is not None else ts[0] if len(ts) == 1 else tuple(ts))
            ring = _ring_part(cfg, l)
            self.rings.append(new(self.num_slots, ring, dtype) if ring else None)
        self.allocator = BlockAllocator(self.num_blocks, reserved=1)
        self.states = BlockAllocator(self.num_slots, reserved=0)

    def __getitem__(self, i):
        return self.layers[i]

    def __len__(self):
        return len(self.layers)

    @property
    def bytes(self) -> int:
        ts = [t for c, l in zip(self.layers, self.cfg.layers) if getattr(l.mixer, "kv_from", None) is None
              for t in (c if isinstance(c, tuple) else (c,))] + self.rings
        ts = [t for t in ts if t is not None and t is not self.plane]
        return sum(t.numel() * t.element_size() for t in ts + ([self.plane] if self.plane is not None else []))

    @property
    def capacity_tokens(self) -> int:
        return (self.num_blocks - 1) * KV_BLOCK

    @staticmethod
    def sizes(cfg: HybridConfig, dtype) -> tuple[int, int]:
        """(bytes of a block over all layers, bytes of a state slot over all layers)."""
        def count(parts):
            return sum(torch.Size(s).numel() * dt.itemsize for s, dt in parts)

        block, slot = _plane_heads(cfg) * KV_BLOCK * 4, 0
        for l in cfg.layers:
            b, s = _layer_parts(l, dtype)
            ring = _ring_part(cfg, l)
            block += count(b)
            slot += count(s) + (count([(ring, dtype)]) if ring else 0)
        return block, slot

    @staticmethod
    def auto_num_blocks(cfg: HybridConfig, num_slots: int, device, dtype=torch.bfloat16,
                        kv_fraction: float = 0.85, reserve_bytes: int = 8 << 30,
                        max_blocks: int | None = None, hbm_budget: float | None = None,
                        weight_bytes: int | None = None, min_blocks: int = 0) -> int:
        """Blocks beside ``num_slots`` state slots (budget: PagedKVCache.auto_num_blocks).  A
        model without attention layers pays nothing for blocks; 1M of them at most."""
        block, slot = HybridCache.sizes(cfg, dtype)
        n = _budget_blocks(cfg.name, block, slot * num_slots, device, kv_fraction, reserve_bytes,
                           max_blocks, hbm_budget, weight_bytes, min_blocks)
        return min(n, 1 << 20) if block == 0 else n
