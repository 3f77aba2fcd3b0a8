"""Decoder-only models whose layers differ in kind (the Ralesun design): latent attention and
channel-wise gated delta-rule mixers, Dynamic Tanh norms, a 32-bit residual stream.

Same interface as :class:`~.transformer.TransformerLM` towards the engine (packed prefill with
decode rows appended, static-shaped decode, the cache it needs), so scheduler, decode graphs
and sampler serve it unchanged.  Differences the engine sees:

  * prompts can be cut anywhere: a portion continues from the cached latents and the sequence's
    recurrent state (``portions``);
  * a sequence holds a state slot beside its cache blocks (engine/kv_cache.py HybridCache).

Layout: every mixer reads its normed input through ONE fused projection whose sections start at
multiples of 8 columns - latent attention [queries | latent, key part], delta rule [q | k | v |
beta | decay rank | gate rank].  In bf16 the residual stream, norms, rotary angles, scores,
decays, step sizes and the recurrent state are 32-bit; projections and activations bf16.  With
dtype float32 everything is.
"""
from __future__ import annotations

from dataclasses import dataclass

import numpy as np
import torch

from .. import ops
from ..parallel.comm import ParallelContext
from .checkpoint import Tensors
from .config import HybridConfig, LatentAttention
from .transformer import DecodeMeta, PrefillMeta


def _pad(n: int, m: int = 8) -> int:
    return -(-n // m) * m


def _fused_rows(sections: list[torch.Tensor]) -> tuple[torch.Tensor, list[int]]:
    """Stack weights by output rows, each section from a multiple of 8 rows; the total padded to
    the 256-row tiles of the prefill GEMM where that costs little.  -> (weight, offsets)."""
    offs, n = [], 0
    for w in sections:
        offs.append(n)
        n += _pad(w.shape[0])
    n = _pad(n, 256) if n >= 2048 else n
    out = sections[0].new_zeros(n, sections[0].shape[1])
    for o, w in zip(offs, sections):
        out[o:o + w.shape[0]] = w
    return out, offs


@dataclass
class Dyt:
    w: torch.Tensor
    b: torch.Tensor
    alpha: float


@dataclass
class HybridStep:
    """Device metadata of a packed step beyond PrefillMeta: the rows by portion for recurrent
    layers (decode rows are portions of one token), the key rows per window for attention."""
    portions: "ops.Portions"
    keys: dict
    q_cu: torch.Tensor
    q_host: list
    tiles: tuple
    qtile: int


class _Shard:
    """The shard fields the engine reads (these models run unsharded)."""

    def __init__(self, cfg: HybridConfig):
        self.hq = self.hkv = max(l.mixer.heads for l in cfg.layers)
        self.vocab, self.tp, self.rank = cfg.vocab_size, 1, 0


class HybridLM:
    portions = True  # prompts may be cut anywhere

    def __init__(self, cfg: HybridConfig, device: torch.device | str = "cpu",
                 pc: ParallelContext | None = None, seed: int = 0,
                 full_then_shard: bool | None = None, dtype=torch.bfloat16,
                 tensors: dict[str, torch.Tensor] | None = None):
        """``tensors``: checkpoint tensors by name; random weights from ``seed`` without."""
        self.pc = pc or ParallelContext.single()
        if self.pc.tp_size != 1 or self.pc.ep_size != 1:
            raise ValueError(f"{cfg.name}: models with mixed layer kinds run on one GPU per replica")
        self.cfg, self.device, self.dtype = cfg, torch.device(device), dtype
        self.sh = _Shard(cfg)
        self.ep_overflow = None
        src = Tensors(tensors) if tensors is not None else _RandomTensors(cfg, seed, self.device)
        self._load(src)
        self._rope: dict = {}
        for l in cfg.layers:
            m = l.mixer
            if isinstance(m, LatentAttention) and (m.rot_base, m.rot_dims) not in self._rope:
                self._rope[m.rot_base, m.rot_dims] = ops.build_interleaved_rope(
                    cfg.max_position, m.rot_dims, m.rot_base, self.device)

    # ------------------------------------------------------------ weights
    def _load(self, src) -> None:
        cfg, dev, dt = self.cfg, self.device, self.dtype
        W = cfg.hidden_size

        def lin(t):
            return t.to(device=dev, dtype=dt).contiguous()

        def f32(t):
            return t.to(device=dev, dtype=torch.float32).contiguous()

        def norm(name):
            return Dyt(f32(src.take(name, W)), f32(src.take(name + ".b", W)),
                       float(src.take(name + ".alpha")))

        self.embed = lin(src.take("embed", cfg.vocab_size, W))
        self.layers = []
        for i, l in enumerate(cfg.layers):
            p, m = f"l{i}.mix.", l.mixer
            L: dict = {"norm1": norm(f"l{i}.norm1")}
            if isinstance(m, LatentAttention):
                w, offs = _fused_rows([src.take(p + "q", m.heads * (m.dim + m.rot_dim), W),
                                       src.take(p + "dkv", m.kv_rank + m.rot_dim, W)])
                L["in"], L["off_kv"] = lin(w), offs[1]
                L["c_norm"] = f32(src.take(p + "dkv.norm", m.kv_rank))
                uk = src.take(p + "uk", m.heads * m.dim, m.kv_rank)
                uv = src.take(p + "uv", m.heads * m.vdim, m.kv_rank)
                w, offs = _fused_rows([uk, uv])
                L["up"], L["voff"] = lin(w), offs[1]
                # decode: per-head key projection transposed (queries into the latent space),
                # per-head value projection as it is
                L["uk_t"] = lin(uk.view(m.heads, m.dim, m.kv_rank).transpose(1, 2))
                L["uv"] = L["up"][offs[1]:offs[1] + m.heads * m.vdim].view(m.heads, m.vdim, m.kv_rank)
                L["sink"] = f32(src.take(p + "sink", m.heads)) if m.sink else None
                L["o"] = lin(src.take(p + "o", W, m.heads * m.vdim))
            else:
                kd, vd = m.kv_heads * m.dim, m.heads * m.vdim
                ra, rg = src.shape(p + "a1")[0], src.shape(p + "g1")[0]
                qkv = torch.cat([src.take(p + "q", kd, W), src.take(p + "k", kd, W),
                                 src.take(p + "v", vd, W)])
                w, offs = _fused_rows([qkv, src.take(p + "b", m.heads, W),
                                       src.take(p + "a1", ra, W), src.take(p + "g1", rg, W)])
                L["in"] = lin(w)
                L["off_b"], L["off_a"], L["off_g"] = offs[1:]
                for k, r, n in (("a2", ra, m.heads * m.dim), ("g2", rg, vd)):
                    w = src.take(p + k, n, r)  # padded ranks: the fused rows there are zero
                    L[k] = lin(torch.nn.functional.pad(w, (0, _pad(r) - r)))
                conv = torch.cat([src.take(p + x + ".conv", n, m.conv)
                                  for x, n in (("q", kd), ("k", kd), ("v", vd))])
                L["delta"] = ops.DeltaWeights(
                    conv=f32(conv.float().t()), a_exp=f32(src.take(p + "A_log", m.heads).float().exp()),
                    dt_bias=f32(src.take(p + "dt_bias", m.heads * m.dim)),
                    norm=f32(src.take(p + "norm", m.vdim)), eps=cfg.norm_eps, heads=m.heads,
                    kv_heads=m.kv_heads, dim=m.dim, vdim=m.vdim)
                L["o"] = lin(src.take(p + "o", W, vd))
            if l.ff:
                q, ffp = f"l{i}.mlp.", _pad(l.ff)
                L["norm2"] = norm(f"l{i}.norm2")
                gu = self.embed.new_zeros(2 * ffp, W)
                gu[:l.ff] = lin(src.take(q + "gate", l.ff, W))
                gu[ffp:ffp + l.ff] = lin(src.take(q + "up", l.ff, W))
                L["gate_up"] = gu
                L["down"] = lin(torch.nn.functional.pad(src.take(q + "down", W, l.ff),
                                                        (0, ffp - l.ff)))
            self.layers.append(L)
        self.final = norm("final.norm")
        self.lm_head = lin(src.take("head", cfg.vocab_size, W))
        src.finish()

    def weight_bytes(self) -> int:
        ts = [self.embed, self.lm_head, self.final.w, self.final.b]
        for L in self.layers:
            for k, v in L.items():
                if isinstance(v, torch.Tensor) and k != "uv":  # uv is a view of "up"
                    ts.append(v)
                elif isinstance(v, Dyt):
                    ts += [v.w, v.b]
                elif isinstance(v, ops.DeltaWeights):
                    ts += [v.conv, v.a_exp, v.dt_bias, v.norm]
        return sum(t.numel() * t.element_size() for t in ts)

    # ------------------------------------------------------------ engine hooks
    def new_cache(self, num_blocks: int, max_batch: int):
        from ..engine.kv_cache import HybridCache

        return HybridCache(self.cfg, num_blocks, max_batch, self.device, self.dtype)

    def auto_num_blocks(self, max_batch: int, **kw) -> int:
        from ..engine.kv_cache import HybridCache

        return HybridCache.auto_num_blocks(self.cfg, max_batch, self.device, self.dtype, **kw)

    def decode_buffer(self, max_batch: int) -> torch.Tensor | None:
        return None

    def decode_meta(self, Bb: int, max_blocks: int, **tensors) -> DecodeMeta:
        """Persistent decode metadata of a batch bucket: split workspaces per geometry."""
        ws = {}
        for l in self.cfg.layers:
            m = l.mixer
            if isinstance(m, LatentAttention):
                key = (m.heads, m.kv_rank, m.window)
                if key not in ws:
                    ws[key] = ops.LatentDecodeWorkspace(Bb, *key, max_blocks, self.device)
        return DecodeMeta(blocks_per_part=0, workspace=ws, **tensors)

    def step_arrays(self, lens: np.ndarray, starts: np.ndarray, blk_tab: np.ndarray,
                    state: np.ndarray, Tp: int, dec_state: np.ndarray,
                    dec_pos: np.ndarray) -> tuple[dict, dict, dict]:
        """Host metadata of a packed step: ``lens`` tokens of each portion from position
        ``starts``, block tables, state slots; prefill rows padded to Tp; decode rows behind.
        -> (int32 arrays, int64 arrays, host values) for :meth:`step_meta`."""
        n, nd = len(lens), len(dec_state)
        cu = np.zeros(n + 1, np.int64)
        np.cumsum(lens, out=cu[1:])
        T, R = int(cu[-1]), Tp + nd
        row_off = np.zeros(R, np.int64)
        row_off[:T] = np.arange(T) - np.repeat(cu[:-1], lens)
        row_state = np.full(R, -1, np.int64)
        row_state[:T] = np.repeat(state, lens)
        row_state[Tp:] = dec_state
        a32 = {"row_off": row_off, "row_state": row_state,
               "seg_row": np.concatenate([cu[:-1], Tp + np.arange(nd)]),
               "seg_len": np.concatenate([lens, np.ones(nd, np.int64)]),
               "seg_pos": np.concatenate([starts, dec_pos]),
               "seg_state": np.concatenate([state, dec_state]), "q_cu": cu}
        a64: dict = {}
        keys = {}
        bs = ops.KV_BLOCK
        for w in self.cfg.windows:
            ctx = np.array([ops.window_reach(int(s), w) for s in starts], np.int64)
            k_cu = np.zeros(n + 1, np.int64)
            np.cumsum(ctx + lens, out=k_cu[1:])
            if ctx.any():
                K = int(k_cu[-1])
                seg = np.repeat(np.arange(n), ctx + lens)
                pos = np.arange(K) - np.repeat(k_cu[:-1], ctx + lens) + (starts - ctx)[seg]
                slots = np.full(_pad(K, 32) if K <= 256 else _pad(K, 256), -1, np.int64)
                slots[:K] = blk_tab[seg, pos // bs] * bs + pos % bs
                a64[f"slots_{w}"] = slots
            a32[f"k_cu_{w}"], a32[f"ctx_{w}"] = k_cu, ctx
            keys[w] = (k_cu.tolist(), ctx.tolist())
        max_len = int(lens.max()) if n else 0
        qtile = 64
        att = [l.mixer for l in self.cfg.layers if isinstance(l.mixer, LatentAttention)]
        if att:
            qtile = min(ops.latent_qtile(max_len, m.dim, m.rot_dim, m.vdim) for m in att)
        ts, tq = ops.portion_tiles(cu.tolist(), qtile)
        a32["tile_seq"], a32["tile_q0"] = np.asarray(ts, np.int64), np.asarray(tq, np.int64)
        return a32, a64, {"q_host": cu.tolist(), "keys": keys, "qtile": qtile, "max_len": max_len}

    def step_meta(self, t32: dict, t64: dict, host: dict) -> HybridStep:
        p = ops.Portions(t32["seg_row"], t32["seg_len"], t32["seg_pos"], t32["seg_state"],
                         t32["row_off"], t32["row_state"], host["max_len"])
        keys = {w: ops.PortionKeys(t32[f"k_cu_{w}"], t32[f"ctx_{w}"], t64.get(f"slots_{w}"), kh, ch)
                for w, (kh, ch) in host["keys"].items()}
        return HybridStep(p, keys, t32["q_cu"], host["q_host"],
                          (t32["tile_seq"], t32["tile_q0"]), host["qtile"])

    # ------------------------------------------------------------ mixers
    def _latent_decode(self, i: int, L: dict, m: LatentAttention, proj, positions, slots, kv,
                       dm: DecodeMeta, out: torch.Tensor) -> None:
        """One token per row of ``proj``, in the latent space -> out [rows, heads * vdim]."""
        cache = kv[i]
        B = proj.shape[0]
        qa = proj.new_empty(B, m.heads, cache.shape[-1])
        ops.latent_prep(proj, L["off_kv"], m.heads, m.dim, m.rot_dim, m.rot_dims, m.kv_rank,
                        L["c_norm"], self.cfg.norm_eps, self._rope[m.rot_base, m.rot_dims],
                        positions, slots, cache, qa=qa)
        dq = m.dim + m.rot_dim
        ops.head_linear(proj[:, :m.heads * dq].unflatten(1, (m.heads, dq)), L["uk_t"], out=qa)
        o = ops.latent_decode_attention(qa, cache, m.kv_rank, dm.block_tables, dm.context_lens,
                                        m.window, m.scale, L["sink"],
                                        dm.workspace[m.heads, m.kv_rank, m.window])
        ops.head_linear(o, L["uv"], out=out.view(B, m.heads, m.vdim))

    def _latent_prefill(self, i: int, L: dict, m: LatentAttention, x, meta: PrefillMeta, kv):
        step: HybridStep = meta.extra
        proj = ops.linear(x, L["in"])
        R, Tp, T = x.shape[0], meta.n_prefill, step.q_host[-1]
        cache = kv[i]
        a = proj.new_empty(R, m.heads * m.vdim)
        lat = proj.new_empty(Tp, cache.shape[-1])
        ops.latent_prep(proj[:Tp], L["off_kv"], m.heads, m.dim, m.rot_dim, m.rot_dims, m.kv_rank,
                        L["c_norm"], self.cfg.norm_eps, self._rope[m.rot_base, m.rot_dims],
                        meta.positions, meta.slots, cache, lat=lat)
        keys = step.keys[m.window]
        if keys.slots is not None:
            lat = ops.latent_gather(cache, keys.slots)
        up = ops.linear(lat[:, :m.kv_rank], L["up"])
        ops.latent_prefill_attention(proj, up, L["voff"], lat, m.kv_rank, m.heads, m.dim,
                                     m.rot_dim, m.vdim, step.q_cu, step.q_host, keys, step.tiles,
                                     step.qtile, m.window, m.scale, L["sink"], a)
        if T < Tp:
            a[T:Tp].zero_()
        if Tp < R:
            self._latent_decode(i, L, m, proj[Tp:], meta.positions[Tp:], meta.slots[Tp:], kv,
                                meta.decode, a[Tp:])
        return a

    def _delta(self, i: int, L: dict, x, kv, meta) -> torch.Tensor:
        w = L["delta"]
        proj = ops.linear(x, L["in"])
        decay = ops.linear(proj[:, L["off_a"]:L["off_a"] + L["a2"].shape[1]], L["a2"])
        gate = ops.linear(proj[:, L["off_g"]:L["off_g"] + L["g2"].shape[1]], L["g2"])
        ring, state = kv[i]
        if isinstance(meta, DecodeMeta):
            return ops.delta_decode(proj, L["off_b"], w, ring, state, decay, gate,
                                    meta.positions, meta.state)
        p = meta.extra.portions
        conv = ops.short_conv(proj, w, ring, meta.positions, p)
        return ops.delta_scan(proj, L["off_b"], conv, w, ring, state, decay, gate, p)

    # ------------------------------------------------------------ forward
    def _run(self, ids: torch.Tensor, mix, rows: torch.Tensor | None = None) -> torch.Tensor:
        """Layer stack on the 32-bit residual stream -> logits.  ``rows``: continue with these
        rows only once the last mixer has read (and cached) every row."""
        cfg, dt = self.cfg, self.dtype
        h = torch.empty((ids.shape[0], cfg.hidden_size), dtype=torch.float32, device=self.device)
        y, last = None, len(self.layers) - 1
        for i, (l, L) in enumerate(zip(cfg.layers, self.layers)):
            n = L["norm1"]
            x = ops.dyt(h, n.w, n.b, n.alpha, y=y, ids=ids if i == 0 else None, embed=self.embed,
                        dtype=dt)
            a = mix(i, l.mixer, L, x)
            if i == last and rows is not None:
                a, h = a.index_select(0, rows), h.index_select(0, rows)
            y = ops.linear(a, L["o"])
            if l.ff:
                n = L["norm2"]
                x = ops.dyt(h, n.w, n.b, n.alpha, y=y, dtype=dt)
                y = ops.linear(ops.gated(x, L["gate_up"], cfg.act), L["down"])
        n = self.final
        return ops.linear(ops.dyt(h, n.w, n.b, n.alpha, y=y, dtype=dt), self.lm_head)

    def forward_prefill(self, ids: torch.Tensor, meta: PrefillMeta, kv) -> torch.Tensor:
        """Packed prompt portions, optionally with decode rows appended; logits of the rows in
        ``meta.last_idx``."""
        def mix(i, m, L, x):
            if isinstance(m, LatentAttention):
                return self._latent_prefill(i, L, m, x, meta, kv)
            return self._delta(i, L, x, kv, meta)

        return self._run(ids, mix, meta.last_idx)

    def forward_decode(self, ids: torch.Tensor, meta: DecodeMeta, kv,
                       attn_out: torch.Tensor | None = None) -> torch.Tensor:
        """One token per sequence; static shapes (graph-capturable)."""
        def mix(i, m, L, x):
            if isinstance(m, LatentAttention):
                proj = ops.linear(x, L["in"])
                a = proj.new_empty(x.shape[0], m.heads * m.vdim)
                self._latent_decode(i, L, m, proj, meta.positions, meta.slots, kv, meta, a)
                return a
            return self._delta(i, L, x, kv, meta)

        return self._run(ids, mix)

    # ------------------------------------------------------------ reference
    def forward_reference(self, ids_list: list[list[int]]) -> list[torch.Tensor]:
        """Whole sequences, each in one pass over a scratch cache -> logits of every position."""
        outs = []
        for ids in ids_list:
            n = len(ids)
            nb = -(-n // ops.KV_BLOCK)
            kv = self.new_cache(nb + 1, 1)
            blocks = np.arange(1, nb + 1)
            a32, a64, host = self.step_arrays(np.array([n]), np.array([0]), blocks[None],
                                              np.array([0]), n, np.zeros(0, np.int64),
                                              np.zeros(0, np.int64))
            dev = self.device
            i32 = {k: torch.as_tensor(v.astype(np.int32), device=dev) for k, v in a32.items()}
            i64 = {k: torch.as_tensor(v, device=dev) for k, v in a64.items()}
            pos = torch.arange(n, dtype=torch.int32, device=dev)
            meta = PrefillMeta(positions=pos,
                               slots=torch.arange(n, dtype=torch.int64, device=dev) + ops.KV_BLOCK,
                               cu_seqlens=i32["q_cu"], cu_host=[0, n], tiles=None,
                               last_idx=torch.arange(n, dtype=torch.int64, device=dev),
                               n_prefill=n, extra=self.step_meta(i32, i64, host))
            outs.append(self.forward_prefill(
                torch.as_tensor(list(ids), dtype=torch.int32, device=dev), meta, kv))
        return outs


class _RandomTensors:
    """Random weights under the checkpoint's names: normal weights of ``init_std``, norms near
    identity, decays spread over slow and fast channels."""

    def __init__(self, cfg: HybridConfig, seed: int, device: torch.device):
        self.cfg = cfg
        gdev = device if cfg.num_params() >= 200_000_000 and device.type == "cuda" else "cpu"
        self.dev = torch.device(gdev)
        self.gen = torch.Generator(device=self.dev).manual_seed(seed)
        self._mixer = {f"l{i}.mix.": l.mixer for i, l in enumerate(cfg.layers)}

    def shape(self, name: str) -> tuple:
        m = self._mixer[name[:name.index("mix.") + 4]]
        rank = (m.decay_rank or m.dim) if name.endswith("a1") else (m.gate_rank or m.vdim)
        return (rank, self.cfg.hidden_size)

    def take(self, name: str, *shape: int) -> torch.Tensor:
        leaf = name.rsplit(".", 1)[-1]
        kw = dict(generator=self.gen, device=self.dev, dtype=torch.float32)
        if leaf == "alpha":
            return torch.tensor(0.8)
        if leaf in ("norm", "norm1", "norm2"):
            t = 1 + 0.1 * torch.randn(*shape, **kw)
        elif leaf == "A_log":
            t = torch.rand(*shape, **kw) * 2 - 1
        elif leaf == "dt_bias":
            t = torch.rand(*shape, **kw) * 6 - 5
        elif leaf == "conv":
            t = torch.randn(*shape, **kw) * shape[1] ** -0.5
        elif leaf in ("sink", "b") and len(shape) == 1:
            t = torch.randn(*shape, **kw) * (1.0 if leaf == "sink" else 0.05)
        elif leaf in ("uk", "uv", "a2", "g2"):
            t = torch.randn(*shape, **kw) * shape[1] ** -0.5
        elif leaf == "embed":
            t = torch.randn(*shape, **kw)
        else:
            t = torch.randn(*shape, **kw) * self.cfg.init_std
        return t.to(torch.bfloat16)

    def finish(self) -> None:
        pass
