"""Decoder-only models whose layers differ in kind: a mixer per layer (models/mixers.py) and a layer
structure.

  serial    norm -> mixer -> add, norm -> gated feed-forward -> add (the Ralesun design: latent
            attention and channel-wise gated delta rule, Dynamic Tanh; the Nurilorn design:
            grouped attention with convolved projections, RMS norms in groups, factors on what
            is added, a clamped feed-forward or routed experts)
  parallel  two layer norms of one stream, each followed by a causal convolution -> mixer and
            squared-relu feed-forward -> one add (the Mebalorn design: talking-heads attention and
            minGRU, sinusoidal positions, capped logits)
  joint     one layer norm -> mixer, squared-relu experts and a shared one -> one add, then a gated
            input of the token to this layer -> norm -> add (the Garesun design: retention, matrix
            memory, latent attention whose latents several layers may share)

Same interface as :class:`~.transformer.TransformerLM` towards the engine (packed prefill with
decode rows appended, static-shaped decode, the cache it needs), so scheduler, decode graphs
and sampler serve it unchanged.  Differences the engine sees:

  * prompts can be cut anywhere: a portion continues from the cached tokens and the sequence's
    recurrent state (``portions``);
  * a sequence holds a state slot beside its cache blocks (engine/kv_cache.py HybridCache).

In bf16 the residual stream, norms, angles, scores, attention weights, decays, step sizes, gates of
a recurrence and its state are 32-bit; projections and activations bf16.  With dtype float32
everything is.  In a parallel or joint layer mixer and (shared) feed-forward write the columns of ONE
operand of ONE output projection, so their sum is formed in its fp32 accumulators.
"""
from __future__ import annotations

from dataclasses import dataclass

import numpy as np
import torch

from .. import ops
from ..parallel.comm import ParallelContext
from .checkpoint import Tensors
from .config import (GatedAverage, GroupedAttention, HybridConfig, LatentAttention,
                     TalkingAttention)
from .mixers import MIXERS, GroupedMixer, TalkingMixer, pad_to
from .transformer import DecodeMeta, PrefillMeta


@dataclass
class Dyt:
    w: torch.Tensor
    b: torch.Tensor
    alpha: float


@dataclass
class GroupNorm:
    w: torch.Tensor


@dataclass
class PlainNorm:
    """Layer norm without bias."""
    w: torch.Tensor


@dataclass
class HybridStep:
    """Device metadata of a packed step beyond PrefillMeta: the rows by portion for recurrent
    layers and convolutions (decode rows are portions of one token), the key rows per window for
    latent attention, the cached blocks for talking heads and grouped attention."""
    portions: "ops.Portions"
    keys: dict
    q_cu: torch.Tensor
    q_host: list
    tiles: tuple
    qtile: int
    talk: "ops.TalkPortions | None" = None
    conv_tiles: "ops.ConvTiles | None" = None
    scan_chunks: "ops.ScanChunks | None" = None
    grouped: "ops.GroupedPortions | None" = None


class _Shard:
    """The shard fields the engine reads (these models run unsharded)."""

    def __init__(self, cfg: HybridConfig):
        self.hq = self.hkv = max(getattr(l.mixer, "heads", 1) for l in cfg.layers)
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
        self._rope: dict = {}
        self._load(src)
        self.moe_ws = None
        moe = [l for l in cfg.layers if l.experts]
        if moe and self.device.type == "cuda":
            # one scratch for every layer, in packed steps and decode graphs
            f32, W = self.dtype == torch.float32, self._moe_width
            n = max(ops.moe.workspace_bytes(ops.moe.MOE_CHUNK, W, self._expert_ff(l.ff),
                                            l.experts.count, l.experts.top, f32) for l in moe)
            ops.gemm.gemm_workspace(self.device)
            self.moe_ws = torch.empty(n, dtype=torch.uint8, device=self.device)

    # ------------------------------------------------------------ weights
    def lin(self, t: torch.Tensor) -> torch.Tensor:
        """A matrix in the activation type."""
        return t.to(device=self.device, dtype=self.dtype).contiguous()

    def f32(self, t: torch.Tensor) -> torch.Tensor:
        return t.to(device=self.device, dtype=torch.float32).contiguous()

    def rope(self, base: float, dims: int, scaling=None) -> torch.Tensor:
        """The rotation table layers of this base, size and scaling share."""
        key = (base, dims, scaling)
        if key not in self._rope:
            self._rope[key] = ops.build_interleaved_rope(self.cfg.max_position, dims, base,
                                                         self.device, scaling)
        return self._rope[key]

    @property
    def _moe_width(self) -> int:
        """Columns of the experts' input and output: the grouped GEMMs of bf16 take multiples of
        128 (zeros behind the width)."""
        W = self.cfg.hidden_size
        return W if self.dtype == torch.float32 else pad_to(W, 128)

    def _expert_ff(self, ff: int) -> int:
        if self.dtype == torch.float32:
            return ff
        return pad_to(ff, 128 if self.cfg.block == "joint" else 64)

    def _norm(self, src, name: str, conv: str | None = None):
        W, t = self.cfg.hidden_size, self.cfg.conv_taps
        if self.cfg.norm == "group_rms":
            w = self.f32(src.take(name, W))
            # the logits' factor rides on the last norm's weights
            return GroupNorm(w * self.cfg.logit_scale if name == "final.norm" else w)
        if self.cfg.norm == "layer":
            return PlainNorm(self.f32(src.take(name, W)))
        w, b = src.take(name, W), src.take(name + ".b", W)
        if self.cfg.block == "serial":
            return Dyt(self.f32(w), self.f32(b), float(src.take(name + ".alpha")))
        c = None if conv is None else self.lin(src.take(conv, W, t).t())
        return ops.LayerNorm(self.lin(w), self.lin(b), c)

    def _load(self, src) -> None:
        cfg, lin, W = self.cfg, self.lin, self.cfg.hidden_size
        parallel = cfg.block == "parallel"
        pad = torch.nn.functional.pad
        self.embed = lin(src.take("embed", cfg.vocab_size, W))
        self.turns = ops.sinusoid_turns(W, self.device) if cfg.sinusoids else None
        scaled = cfg.norm == "group_rms"
        self.layers = []
        for i, l in enumerate(cfg.layers if cfg.block == "joint" else ()):
            self.layers.append(self._load_joint(src, i, l))
        if cfg.side_dim:
            self.side_embed = lin(src.take("side.embed", cfg.vocab_size, cfg.num_layers * cfg.side_dim))
        for i, l in enumerate(cfg.layers if cfg.block != "joint" else ()):
            p, q = f"l{i}.", f"l{i}.mlp."
            mixer = MIXERS[type(l.mixer)](l.mixer, p + "mix.", src, self)
            L: dict = {"norm1": self._norm(src, p + "norm1", p + "canon1"), "mixer": mixer}
            for k in (1, 2) if scaled and l.ff else (1,) if scaled else ():
                L[f"add{k}"] = self.f32(src.take(f"{p}ls{k}", W)) * cfg.residual_mult
            ffp = pad_to(l.ff) if l.ff else 0
            if scaled and not l.ff:
                src.discard(p + "norm2")
                src.discard(p + "ls2")
            if l.experts:
                L["norm2"] = self._norm(src, p + "norm2")
                self._load_experts(src, q, l, L)
            elif l.ff:
                L["norm2"] = self._norm(src, p + "norm2", p + "canon2")
                down = lin(pad(src.take(q + "down", W, l.ff), (0, ffp - l.ff)))
                up = lin(src.take(q + "up", l.ff, W))
                if parallel:
                    L["up"] = pad(up, (0, 0, 0, ffp - l.ff)).contiguous()
                else:
                    L["down"] = down
                    L["gate_up"] = self.embed.new_zeros(2 * ffp, W)
                    L["gate_up"][:l.ff] = lin(src.take(q + "gate", l.ff, W))
                    L["gate_up"][ffp:ffp + l.ff] = up
            if parallel:  # [mixer | feed-forward] columns of one output projection
                L["out"] = torch.cat([mixer.o, down], 1).contiguous() if l.ff else mixer.o
                mixer.o = None
            self.layers.append(L)
        self.final = self._norm(src, "final.norm")
        self.lm_head = lin(src.take("head", cfg.vocab_size, W))
        src.finish()

    def _load_joint(self, src, i: int, l) -> dict:
        cfg, lin, W = self.cfg, self.lin, self.cfg.hidden_size
        p, q = f"l{i}.", f"l{i}.mlp."
        mixer = MIXERS[type(l.mixer)](l.mixer, p + "mix.", src, self)
        L: dict = {"norm1": self._norm(src, p + "norm1"), "mixer": mixer}
        # the feed-forward every token uses writes behind the mixer: [mixer | feed-forward] columns
        # of one output projection
        name, ff = (q + "shared.", l.shared) if l.experts else (q, l.ff)
        off, ffp = pad_to(mixer.width), pad_to(ff or 0)
        L["out"] = self.embed.new_zeros(W, off + ffp)
        L["out"][:, :mixer.width] = mixer.o
        mixer.o = None
        if ff:
            L["up"] = self.embed.new_zeros(ffp, W)
            L["up"][:ff] = lin(src.take(name + "up", ff, W))
            L["out"][:, off:off + ff] = lin(src.take(name + "down", W, ff))
        if l.experts:
            self._load_experts(src, q, l, L)
        if cfg.side_dim:
            L["side_gate"] = lin(src.take(p + "side.gate", cfg.side_dim, W))
            L["side_proj"] = lin(src.take(p + "side.proj", W, cfg.side_dim))
            L["side_norm"] = self.f32(src.take(p + "side.norm", W))
        return L

    def _load_experts(self, src, q: str, l, L: dict) -> None:
        W, ff, n = self.cfg.hidden_size, l.ff, l.experts.count
        Wp, fp = self._moe_width, self._expert_ff(ff)
        new, gated = self.embed.new_zeros, self.cfg.act != "relu2"
        L["experts_in"], L["experts_out"] = new(n, (1 + gated) * fp, Wp), new(n, Wp, fp)
        for e in range(n):
            if gated:
                L["experts_in"][e, :ff, :W] = self.lin(src.take(f"{q}e{e}.gate", ff, W))
            up = fp if gated else 0
            L["experts_in"][e, up:up + ff, :W] = self.lin(src.take(f"{q}e{e}.up", ff, W))
            L["experts_out"][e, :W, :ff] = self.lin(src.take(f"{q}e{e}.down", W, ff))
        L["router"] = new(n, Wp)
        L["router"][:, :W] = self.lin(src.take(q + "router", n, W))

    def weight_bytes(self) -> int:
        def norm(n):
            return [t for t in vars(n).values() if isinstance(t, torch.Tensor)]

        ts = [self.embed, self.lm_head, *norm(self.final)]
        ts += [self.side_embed] if self.cfg.side_dim else []
        for L in self.layers:
            for v in L.values():
                ts += [v] if isinstance(v, torch.Tensor) else \
                    norm(v) if isinstance(v, (Dyt, GroupNorm, PlainNorm, ops.LayerNorm)) else v.operands()
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
            elif isinstance(m, TalkingAttention):
                key = TalkingMixer.workspace_key(m)
                if key not in ws:
                    ws[key] = ops.TalkDecodeWorkspace(Bb, *key[1:], max_blocks, self.device)
            elif isinstance(m, GroupedAttention):
                key = GroupedMixer.workspace_key(m)
                if key not in ws:
                    ws[key] = ops.GroupedDecodeWorkspace(Bb, *key[1:], max_blocks, self.device)
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
                slots = np.full(pad_to(K, 32) if K <= 256 else pad_to(K, 256), -1, np.int64)
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
        host: dict = {"starts": starts.tolist(), "conv_per": 0, "qtiles": {}}
        for m in (l.mixer for l in self.cfg.layers if isinstance(l.mixer, GroupedAttention)):
            rep = m.heads // m.kv_heads
            t = ops.grouped_qtile(max_len * rep, m.dim, m.vdim)
            host["qtiles"][rep] = min(t, host["qtiles"].get(rep, t))
        for rep, t in host["qtiles"].items():
            seq, row = _runs(lens * rep, t)
            order = np.argsort(-(starts[seq] * rep + row), kind="stable")  # most keys first
            a32[f"rows_seq_{rep}"], a32[f"rows_at_{rep}"] = seq[order], row[order]
            a32["blocks"] = blk_tab.reshape(-1)
        if any(isinstance(l.mixer, TalkingAttention) for l in self.cfg.layers):
            for name, rows in (("mix", ops.MIX_TILE), ("stats", ops.STATS_TILE)):
                seq, q0 = _runs(lens, rows)
                order = np.argsort(-(starts[seq] + q0), kind="stable")  # most keys first
                a32[name + "_seq"], a32[name + "_q0"] = seq[order], q0[order]
            a32["blocks"] = blk_tab.reshape(-1)
        average = [l.mixer.width for l in self.cfg.layers if isinstance(l.mixer, GatedAverage)]
        if average and ops.chunk_scan(a32["seg_len"], max(average)):
            a32["scan_seg"], a32["scan_off"] = _runs(a32["seg_len"], ops.SCAN_CHUNK)
        if self.cfg.taps > 1 or host["qtiles"]:
            tile_rows = ops.prep_tile_rows if host["qtiles"] else ops.conv_tile_rows
            host["conv_per"] = tile_rows(R, self.cfg.taps)
            a32["conv_seg"], a32["conv_off"] = _runs(a32["seg_len"], host["conv_per"])
        return a32, a64, {**host, "q_host": cu.tolist(), "keys": keys, "qtile": qtile,
                          "max_len": max_len}

    def step_meta(self, t32: dict, t64: dict, host: dict) -> HybridStep:
        p = ops.Portions(t32["seg_row"], t32["seg_len"], t32["seg_pos"], t32["seg_state"],
                         t32["row_off"], t32["row_state"], host["max_len"])
        keys = {w: ops.PortionKeys(t32[f"k_cu_{w}"], t32[f"ctx_{w}"], t64.get(f"slots_{w}"), kh, ch)
                for w, (kh, ch) in host["keys"].items()}
        talk = conv = grouped = None
        n = len(host["starts"])
        if host["qtiles"]:
            grouped = ops.GroupedPortions(
                t32["q_cu"], t32["seg_pos"][:n], t32["blocks"].view(n, -1),
                {r: (t32[f"rows_seq_{r}"], t32[f"rows_at_{r}"], t) for r, t in host["qtiles"].items()},
                host["q_host"], host["starts"])
        if "mix_seq" in t32:
            talk = ops.TalkPortions(t32["q_cu"], t32["seg_pos"][:n], t32["blocks"].view(n, -1),
                                    (t32["mix_seq"], t32["mix_q0"]),
                                    (t32["stats_seq"], t32["stats_q0"]), host["q_host"], host["starts"])
        scan = ops.ScanChunks(t32["scan_seg"], t32["scan_off"]) if "scan_seg" in t32 else None
        if host["conv_per"]:
            conv = ops.ConvTiles(t32["conv_seg"], t32["conv_off"], host["conv_per"])
        return HybridStep(p, keys, t32["q_cu"], host["q_host"],
                          (t32["tile_seq"], t32["tile_q0"]), host["qtile"], talk, conv, scan,
                          grouped)

    # ------------------------------------------------------------ forward
    def _serial(self, ids: torch.Tensor, mix, rows: torch.Tensor | None) -> torch.Tensor:
        """Layer stack on the 32-bit residual stream -> logits.  ``rows``: continue with these
        rows only once the last mixer has read (and cached) every row."""
        cfg = self.cfg
        h = torch.empty((ids.shape[0], cfg.hidden_size), dtype=torch.float32, device=self.device)
        y, by, last = None, None, len(self.layers) - 1
        for i, (l, L) in enumerate(zip(cfg.layers, self.layers)):
            x = self._enter(L["norm1"], h, y, by, ids=ids if i == 0 else None)
            a = mix(i, L["mixer"], x)
            if i == last and rows is not None:
                a, h = a.index_select(0, rows), h.index_select(0, rows)
            y, by = ops.linear(a, L["mixer"].o), L.get("add1")
            if l.experts:
                x = self._enter(L["norm2"], h, y, by, width=self._moe_width)
                y, by = self._experts(L, l, x), L["add2"]
            elif l.ff:
                x = self._enter(L["norm2"], h, y, by)
                y = ops.linear(ops.gated(x, L["gate_up"], cfg.act, l.limit), L["down"])
                by = L.get("add2")
        return ops.linear(self._enter(self.final, h, y, by), self.lm_head)

    def _enter(self, n, h, y, by, ids=None, width=None) -> torch.Tensor:
        """Norm ``n`` of the stream h after the add of y (times ``by``), or from the embedding."""
        if isinstance(n, Dyt):
            return ops.dyt(h, n.w, n.b, n.alpha, y=y, ids=ids, embed=self.embed, dtype=self.dtype)
        cfg = self.cfg
        return ops.group_rms(h, n.w, cfg.norm_groups, cfg.norm_eps, y=y, scale=by, ids=ids,
                             embed=self.embed, embed_scale=cfg.embed_scale, width=width,
                             dtype=self.dtype)

    def _experts(self, L: dict, l, x: torch.Tensor, **kw) -> torch.Tensor:
        e = l.experts
        return ops.fused_moe(x, ops.router_logits_f32(x, L["router"]), L["experts_in"],
                             L["experts_out"], e.top, self.cfg.act, e.count, workspace=self.moe_ws,
                             groups=e.groups, keep=e.keep, limit=l.limit, **kw)

    def _parallel(self, ids: torch.Tensor, mix, rows: torch.Tensor | None, positions, kv,
                  **where) -> torch.Tensor:
        """As _serial; ``where``: the portions and tiles of a packed step, or the state slots of a
        decode step."""
        cfg, dt, eps, R = self.cfg, self.dtype, self.cfg.norm_eps, ids.shape[0]
        h, y, last = None, None, len(self.layers) - 1
        # rows of one portion read each other's stream while others write theirs: two buffers
        streams = [torch.empty((R, cfg.hidden_size), dtype=torch.float32, device=self.device)
                   for _ in range(2 if "portions" in where else 1)]
        for i, (l, L) in enumerate(zip(cfg.layers, self.layers)):
            norms = [L["norm1"]] + ([L["norm2"]] if l.ff else [])
            first = {"ids": ids, "embed": self.embed, "turns": self.turns} if i == 0 else {}
            xs = ops.norm_conv(norms, eps, h, y=y, positions=positions, ring=kv.rings[i],
                               h_out=streams[i % len(streams)], dtype=dt, **first, **where)
            h = streams[i % len(streams)]
            mw = L["mixer"].width
            a = torch.empty((R, L["out"].shape[1]), dtype=dt, device=self.device)
            mix(i, L["mixer"], xs[0], a[:, :mw])
            if i == last and rows is not None:
                h, part = h.index_select(0, rows), a[:, :mw].index_select(0, rows)
                a = a.new_empty(rows.shape[0], a.shape[1])
                a[:, :mw] = part
                xs = [x.index_select(0, rows) for x in xs]
            if l.ff:
                ops.squared_relu(xs[1], L["up"], a[:, mw:])
            y = ops.linear(a, L["out"])
        x, = ops.norm_conv([self.final], eps, h, y=y, dtype=dt)
        logits = ops.linear(x, self.lm_head)
        return ops.softcap_(logits, cfg.logit_softcap) if cfg.logit_softcap else logits

    def _joint(self, ids: torch.Tensor, mix, rows: torch.Tensor | None) -> torch.Tensor:
        """As _serial: one norm for both sublayers, one add, then the token's input to the layer."""
        cfg, dt, eps, W = self.cfg, self.dtype, self.cfg.norm_eps, self.cfg.hidden_size
        h = torch.empty((ids.shape[0], W), dtype=torch.float32, device=self.device)
        z, zn, last = None, None, len(self.layers) - 1
        for i, (l, L) in enumerate(zip(cfg.layers, self.layers)):
            first = {"ids": ids, "embed": self.embed, "embed_scale": cfg.embed_scale} if i == 0 else {}
            wide = ops.side_norm(h, L["norm1"].w, eps, z, zn, dtype=dt,
                                 width=self._moe_width if l.experts else None, **first)
            x, mw, off = wide[:, :W], L["mixer"].width, pad_to(L["mixer"].width)
            a = torch.empty((ids.shape[0], L["out"].shape[1]), dtype=dt, device=self.device)
            if off > mw:
                a[:, mw:off].zero_()
            mix(i, L["mixer"], x, a[:, :mw])
            if i == last and rows is not None:
                ids, h, a, wide = (t.index_select(0, rows) for t in (ids, h, a, wide))
                x = wide[:, :W]
            if "up" in L:
                ops.squared_relu(x, L["up"], a[:, off:])
            y = ops.linear(a, L["out"])
            if l.experts:
                x = self._experts(L, l, wide, stream=h, y=y)
            else:
                x = ops.stream_add(h, y)
            z = zn = None
            if cfg.side_dim:
                g = ops.side_input(x, L["side_gate"], self.side_embed, ids, i)
                z, zn = ops.linear(g, L["side_proj"]), L["side_norm"]
        return ops.linear(ops.side_norm(h, self.final.w, eps, z, zn, dtype=dt), self.lm_head)

    def forward_prefill(self, ids: torch.Tensor, meta: PrefillMeta, kv) -> torch.Tensor:
        """Packed prompt portions, optionally with decode rows appended; logits of the rows in
        ``meta.last_idx``."""
        carry: dict = {}

        def mix(i, mixer, x, out=None):
            return mixer.prefill(x, meta, kv[i], out, carry)

        if self.cfg.block != "parallel":
            return (self._joint if self.cfg.block == "joint" else self._serial)(ids, mix, meta.last_idx)
        step: HybridStep = meta.extra
        return self._parallel(ids, mix, meta.last_idx, meta.positions, kv, portions=step.portions,
                              tiles=step.conv_tiles)

    def forward_decode(self, ids: torch.Tensor, meta: DecodeMeta, kv,
                       attn_out: torch.Tensor | None = None) -> torch.Tensor:
        """One token per sequence; static shapes (graph-capturable)."""
        carry: dict = {}

        def mix(i, mixer, x, out=None):
            return mixer.decode(x, meta, kv[i], out, carry)

        if self.cfg.block != "parallel":
            return (self._joint if self.cfg.block == "joint" else self._serial)(ids, mix, None)
        return self._parallel(ids, mix, None, meta.positions, kv, row_state=meta.state)

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


def _runs(lens: np.ndarray, rows: int) -> tuple[np.ndarray, np.ndarray]:
    """Runs of at most ``rows`` tokens of sequences of ``lens``: (sequence, first token)."""
    n = -(-lens // rows)
    seq = np.repeat(np.arange(len(lens)), n)
    return seq, (np.arange(int(n.sum())) - np.repeat(np.cumsum(n) - n, n)) * rows


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
        if leaf == "vmix":
            return torch.tensor(0.4)
        if leaf in ("ls1", "ls2"):
            t = 0.8 + 0.1 * torch.randn(*shape, **kw)
        elif leaf in ("norm", "norm1", "norm2"):
            t = 1 + 0.1 * torch.randn(*shape, **kw)
        elif leaf == "A_log":
            t = torch.rand(*shape, **kw) * 2 - 1
        elif leaf == "dt_bias":
            t = torch.rand(*shape, **kw) * 6 - 5
        elif leaf == "talk":
            t = torch.eye(shape[0], device=self.dev) + torch.randn(*shape, **kw) * 0.2 * shape[0] ** -0.5
        elif leaf in ("conv", "canon1", "canon2"):
            t = torch.randn(*shape, **kw) * shape[1] ** -0.5
        elif leaf in ("sink", "b") and len(shape) == 1:
            t = torch.randn(*shape, **kw) * (1.0 if leaf == "sink" else 0.05)
            if name.endswith(".mix.z.b"):  # gates from a few tokens to thousands
                t = t * 40 - 3
            elif name.endswith(".mix.f.b"):
                t = t * 20 + 5
        elif leaf in ("uk", "uv", "a2", "g2"):
            t = torch.randn(*shape, **kw) * shape[1] ** -0.5
        elif leaf == "embed":
            t = torch.randn(*shape, **kw)
        else:
            t = torch.randn(*shape, **kw) * self.cfg.init_std
        return t.to(torch.bfloat16)

    def discard(self, name: str) -> None:
        pass

    def finish(self) -> None:
        pass
