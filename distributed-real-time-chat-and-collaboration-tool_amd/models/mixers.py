"""Token mixers of models with mixed layer kinds (models/hybrid.py), one class per kind of spec in
models/config.py: their weights, and how they run in packed steps and in decode steps.

A mixer reads its (normed) input through ONE fused projection whose sections start at multiples of
8 columns, and writes ``width`` columns - of a buffer of its own, or (``out``) of a wider operand -
that the output projection ``o`` [hidden, width] consumes:

  latent attention   [queries | latent, key part | head gates]
  delta rule         [q | k | v | beta | decay rank | gate rank]
  talking heads      [queries | keys | values], heads padded to multiples of 8
  gated average      [gate | candidate | read-out gate]
  grouped attention  [queries | keys | values | head gates], heads padded to multiples of 8
  retention          [q | k | v | read-out gate]
  matrix memory      [q | k | v | read-out gate | input gates | forget gates]

``carry``: a dict that lives as long as the step, for what layers hand to later ones.
"""
from __future__ import annotations

import torch

from .. import ops
from .config import (ChannelDelta, GatedAverage, GroupedAttention, LatentAttention, MatrixMemory,
                     Retention, TalkingAttention)


def pad_to(n: int, m: int = 8) -> int:
    return -(-n // m) * m


def fused_rows(sections: list[torch.Tensor]) -> tuple[torch.Tensor, list[int]]:
    """Stack weights by output rows, each section from a multiple of 8 rows; the total padded to
    the 256-row tiles of the prefill GEMM where that costs little.  -> (weight, offsets)."""
    offs, n = [], 0
    for w in sections:
        offs.append(n)
        n += pad_to(w.shape[0])
    n = pad_to(n, 256) if n >= 2048 else n
    out = sections[0].new_zeros(n, sections[0].shape[1])
    for o, w in zip(offs, sections):
        out[o:o + w.shape[0]] = w
    return out, offs


def _pad_heads(t: torch.Tensor, heads: int, dim: int) -> torch.Tensor:
    """Rows [heads * dim, ...] with every head padded to a multiple of 8."""
    x = t.reshape(heads, dim, *t.shape[1:])
    return torch.cat([x, x.new_zeros(heads, pad_to(dim) - dim, *t.shape[1:])], 1).flatten(0, 1)


class Mixer:
    """``proj``: the fused input projection; ``o``: the output projection; ``width``: columns
    between them."""
    proj: torch.Tensor
    o: torch.Tensor
    width: int

    def prefill(self, x, meta, cache, out=None, carry=None) -> torch.Tensor:
        """Packed portions (and decode rows behind them): ``meta`` a PrefillMeta."""
        raise NotImplementedError

    def decode(self, x, meta, cache, out=None, carry=None) -> torch.Tensor:
        """One token per sequence: ``meta`` a DecodeMeta."""
        raise NotImplementedError

    def operands(self) -> list[torch.Tensor]:
        ts = []
        for v in vars(self).values():
            ts += [v] if isinstance(v, torch.Tensor) else \
                [t for t in vars(v).values() if isinstance(t, torch.Tensor)] \
                if isinstance(v, (ops.DeltaWeights, ops.TalkWeights, ops.AverageWeights,
                                  ops.GroupedWeights, ops.MemoryWeights)) else []
        return ts

    def _out(self, x, out) -> torch.Tensor:
        return x.new_empty(x.shape[0], self.width) if out is None else out


class LatentMixer(Mixer):
    def __init__(self, m: LatentAttention, p: str, src, model):
        W, lin, f32 = model.cfg.hidden_size, model.lin, model.f32
        self.m, self.eps, self.rope = m, model.cfg.norm_eps, model.rope(m.rot_base, m.rot_dims)
        # whose latents are read: this layer's own, or another's
        self.source = int(p[1:p.index(".")]) if m.kv_from is None else m.kv_from
        own = m.kv_from is None
        sections = [src.take(p + "q", m.heads * (m.dim + m.rot_dim), W)]
        if own:
            sections.append(src.take(p + "dkv", m.kv_rank + m.rot_dim, W))
        if m.gate:
            sections.append(src.take(p + "g", m.heads, W))
        w, offs = fused_rows(sections)
        self.proj, self.off_kv = lin(w), offs[1] if own else None
        self.off_g = offs[-1] if m.gate else None
        self.c_norm = f32(src.take(p + "dkv.norm", m.kv_rank)) if own else None
        uk = src.take(p + "uk", m.heads * m.dim, m.kv_rank)
        uv = src.take(p + "uv", m.heads * m.vdim, m.kv_rank)
        w, offs = fused_rows([uk, uv])
        self.up, self.voff = lin(w), offs[1]
        # decode: per-head key projection transposed (queries into the latent space),
        # per-head value projection as it is
        self.uk_t = lin(uk.view(m.heads, m.dim, m.kv_rank).transpose(1, 2))
        self.uv = self.up[offs[1]:offs[1] + m.heads * m.vdim].view(m.heads, m.vdim, m.kv_rank)
        self.sink = f32(src.take(p + "sink", m.heads)) if m.sink else None
        self.width = m.heads * m.vdim
        self.o = lin(src.take(p + "o", W, self.width))

    def operands(self):
        return [t for t in super().operands() if t is not self.uv and t is not self.rope]

    def _gate(self, proj):
        return None if self.off_g is None else proj[:, self.off_g:self.off_g + self.m.heads]

    def _decode(self, proj, positions, slots, cache, dm, out) -> None:
        """One token per row of ``proj``, in the latent space -> out [rows, heads * vdim]."""
        m = self.m
        B = proj.shape[0]
        qa = proj.new_empty(B, m.heads, cache.shape[-1])
        ops.latent_prep(proj, self.off_kv, m.heads, m.dim, m.rot_dim, m.rot_dims, m.kv_rank,
                        self.c_norm, self.eps, self.rope, positions, slots, cache, qa=qa)
        dq = m.dim + m.rot_dim
        ops.head_linear(proj[:, :m.heads * dq].unflatten(1, (m.heads, dq)), self.uk_t, out=qa)
        o = ops.latent_decode_attention(qa, cache, m.kv_rank, dm.block_tables, dm.context_lens,
                                        m.window, m.scale, self.sink,
                                        dm.workspace[m.heads, m.kv_rank, m.window], self._gate(proj))
        ops.head_linear(o, self.uv, out=out.unflatten(1, (m.heads, m.vdim)))

    def _latents(self, proj, meta, cache, carry):
        """Latent rows of the portions' keys; queries are rotated in place.  Layers that read the
        same cache share them."""
        m, step = self.m, meta.extra
        keys, Tp = step.keys[m.window], meta.n_prefill
        lat = proj.new_empty(Tp, cache.shape[-1]) if self.off_kv is not None else None
        ops.latent_prep(proj[:Tp], self.off_kv, m.heads, m.dim, m.rot_dim, m.rot_dims, m.kv_rank,
                        self.c_norm, self.eps, self.rope, meta.positions, meta.slots, cache, lat=lat)
        if lat is not None:
            carry["latents", self.source] = lat
        if keys.slots is None:
            return carry["latents", self.source]
        if (self.source, m.window) not in carry:
            carry[self.source, m.window] = ops.latent_gather(cache, keys.slots)
        return carry[self.source, m.window]

    def prefill(self, x, meta, cache, out=None, carry=None):
        m, step = self.m, meta.extra
        proj = ops.linear(x, self.proj)
        R, Tp, T = x.shape[0], meta.n_prefill, step.q_host[-1]
        a = self._out(x, out)
        lat = self._latents(proj, meta, cache, carry)
        up = ops.linear(lat[:, :m.kv_rank], self.up)
        ops.latent_prefill_attention(proj, up, self.voff, lat, m.kv_rank, m.heads, m.dim,
                                     m.rot_dim, m.vdim, step.q_cu, step.q_host, step.keys[m.window],
                                     step.tiles, step.qtile, m.window, m.scale, self.sink, a,
                                     self._gate(proj))
        if T < Tp:
            a[T:Tp].zero_()
        if Tp < R:
            self._decode(proj[Tp:], meta.positions[Tp:], meta.slots[Tp:], cache, meta.decode, a[Tp:])
        return a

    def decode(self, x, meta, cache, out=None, carry=None):
        a = self._out(x, out)
        self._decode(ops.linear(x, self.proj), meta.positions, meta.slots, cache, meta, a)
        return a


class DeltaMixer(Mixer):
    def __init__(self, m: ChannelDelta, p: str, src, model):
        W, lin, f32 = model.cfg.hidden_size, model.lin, model.f32
        kd, vd = m.kv_heads * m.dim, m.heads * m.vdim
        ra, rg = src.shape(p + "a1")[0], src.shape(p + "g1")[0]
        qkv = torch.cat([src.take(p + "q", kd, W), src.take(p + "k", kd, W),
                         src.take(p + "v", vd, W)])
        w, offs = fused_rows([qkv, src.take(p + "b", m.heads, W),
                              src.take(p + "a1", ra, W), src.take(p + "g1", rg, W)])
        self.proj = lin(w)
        self.off_b, self.off_a, self.off_g = offs[1:]
        # padded ranks: the fused rows there are zero
        self.a2, self.g2 = (lin(torch.nn.functional.pad(src.take(p + k, n, r), (0, pad_to(r) - r)))
                            for k, r, n in (("a2", ra, m.heads * m.dim), ("g2", rg, vd)))
        conv = torch.cat([src.take(p + x + ".conv", n, m.conv)
                          for x, n in (("q", kd), ("k", kd), ("v", vd))])
        self.w = ops.DeltaWeights(
            conv=f32(conv.float().t()), a_exp=f32(src.take(p + "A_log", m.heads).float().exp()),
            dt_bias=f32(src.take(p + "dt_bias", m.heads * m.dim)),
            norm=f32(src.take(p + "norm", m.vdim)), eps=model.cfg.norm_eps, heads=m.heads,
            kv_heads=m.kv_heads, dim=m.dim, vdim=m.vdim)
        self.width = vd
        self.o = lin(src.take(p + "o", W, vd))

    def _project(self, x):
        proj = ops.linear(x, self.proj)
        decay = ops.linear(proj[:, self.off_a:self.off_a + self.a2.shape[1]], self.a2)
        gate = ops.linear(proj[:, self.off_g:self.off_g + self.g2.shape[1]], self.g2)
        return proj, decay, gate

    def prefill(self, x, meta, cache, out=None, carry=None):
        ring, state = cache
        proj, decay, gate = self._project(x)
        p = meta.extra.portions
        conv = ops.short_conv(proj, self.w, ring, meta.positions, p)
        a = ops.delta_scan(proj, self.off_b, conv, self.w, ring, state, decay, gate, p)
        return a if out is None else out.copy_(a)

    def decode(self, x, meta, cache, out=None, carry=None):
        ring, state = cache
        proj, decay, gate = self._project(x)
        a = ops.delta_decode(proj, self.off_b, self.w, ring, state, decay, gate, meta.positions,
                             meta.state)
        return a if out is None else out.copy_(a)


class TalkingMixer(Mixer):
    def __init__(self, m: TalkingAttention, p: str, src, model):
        W, lin, f32 = model.cfg.hidden_size, model.lin, model.f32
        H, G, d, dv = m.heads, m.kv_heads, m.dim, m.vdim
        w, offs = fused_rows([_pad_heads(src.take(p + x, n * k, W), n, k)
                              for x, n, k in (("q", H, d), ("k", G, d), ("v", G, dv))])
        self.proj, (_, self.off_k, self.off_v) = lin(w), offs
        bias = {x: f32(_pad_heads(src.take(p + x + ".b", n * k), n, k))
                for x, n, k in (("q", H, d), ("k", G, d), ("v", G, dv))}
        norm = {x: f32(_pad_heads(src.take(p + x + ".norm", d), 1, d)) for x in "qk"}
        self.w = ops.TalkWeights(
            bias["q"], bias["k"], bias["v"], norm["q"], norm["k"], f32(src.take(p + "talk", H, H)),
            f32(src.take(p + "sink", H)) if m.sink else None, model.cfg.norm_eps, m.scale, H, G, d, dv)
        self.width = H * self.w.vdimp
        o = src.take(p + "o", W, H * dv)
        self.o = lin(_pad_heads(o.t(), H, dv).t())

    def prefill(self, x, meta, cache, out=None, carry=None):
        k, v, plane = cache
        step = meta.extra
        a = self._out(x, out)
        R, Tp, T = x.shape[0], meta.n_prefill, step.q_host[-1]
        q = ops.head_prep(ops.linear(x, self.proj), self.off_k, self.off_v, self.w, meta.slots, k, v)
        ops.talk_prefill(q[:Tp], k, v, self.w, step.talk, a[:Tp])
        if T < Tp:
            a[T:Tp].zero_()
        if Tp < R:
            self._decode(q[Tp:], meta.decode, cache, a[Tp:])
        return a

    def _decode(self, q, dm, cache, out) -> None:
        k, v, plane = cache
        ops.talk_decode(q, k, v, self.w, plane, dm.block_tables, dm.context_lens,
                        dm.workspace.get(self.workspace_key(self.w)), out)

    @staticmethod
    def workspace_key(m) -> tuple:
        return ("talk", m.heads, m.kv_heads, m.vdim)

    def decode(self, x, meta, cache, out=None, carry=None):
        k, v, _ = cache
        a = self._out(x, out)
        q = ops.head_prep(ops.linear(x, self.proj), self.off_k, self.off_v, self.w, meta.slots, k, v)
        self._decode(q, meta, cache, a)
        return a


class AverageMixer(Mixer):
    def __init__(self, m: GatedAverage, p: str, src, model):
        W, lin, f32, C = model.cfg.hidden_size, model.lin, model.f32, m.width
        pad = pad_to(C) - C
        w, offs = fused_rows([src.take(p + x, C, W) for x in "zxg"])
        self.proj = lin(w)
        zb, xb = (f32(torch.nn.functional.pad(src.take(p + x + ".b", C), (0, pad))) for x in "zx")
        self.w = ops.AverageWeights(zb, xb, offs[1], offs[2])
        self.width = C + pad
        self.o = lin(torch.nn.functional.pad(src.take(p + "o", W, C), (0, pad)))

    def prefill(self, x, meta, cache, out=None, carry=None):
        a = self._out(x, out)
        ops.gated_scan(ops.linear(x, self.proj), self.w, cache, meta.extra.portions, a,
                       meta.extra.scan_chunks)
        return a

    def decode(self, x, meta, cache, out=None, carry=None):
        a = self._out(x, out)
        ops.gated_decode(ops.linear(x, self.proj), self.w, cache, meta.positions, meta.state, a)
        return a


class GroupedMixer(Mixer):
    def __init__(self, m: GroupedAttention, p: str, src, model):
        W, lin, f32 = model.cfg.hidden_size, model.lin, model.f32
        H, G, d, dv = m.heads, m.kv_heads, m.dim, m.vdim
        parts = (("q", H, d), ("k", G, d), ("v", G, dv))
        sections = [_pad_heads(src.take(p + x, n * k, W), n, k) for x, n, k in parts]
        if m.gate:
            sections.append(src.take(p + "g", H, W))
        w, offs = fused_rows(sections)
        self.proj, (_, self.off_k, self.off_v) = lin(w), offs[:3]
        self.off_g = offs[3] if m.gate else None
        if m.conv:
            conv = torch.cat([_pad_heads(src.take(f"{p}{x}.conv", n * k, m.conv), n, k)
                              for x, n, k in parts])
        else:
            conv = torch.ones((H + G) * pad_to(d) + G * pad_to(dv), 1)
        self.rope = model.rope(m.rot_base, m.rot_dims, m.rot_scaling)
        self.v_mix = m.v_mix
        lam = float(src.take(p + "vmix")) if m.v_mix else 0.0
        if not m.v_mix:
            src.discard(p + "vmix")
        self.w = ops.GroupedWeights(f32(conv.float().t()), H, G, d, dv, m.scale, m.rot_dims,
                                    m.softcap, m.sink, lam)
        self.width = H * self.w.vdimp
        self.o = lin(_pad_heads(src.take(p + "o", W, H * dv).t(), H, dv).t())

    def operands(self):
        return [t for t in super().operands() if t is not self.rope]

    @staticmethod
    def workspace_key(m) -> tuple:
        return ("grouped", m.heads, m.kv_heads, m.vdim)

    def _prep(self, x, meta, cache, carry, **rows):
        """-> (queries, gate inputs); keys and values are in the cache."""
        k, v, ring = cache
        proj = ops.linear(x, self.proj)
        first, mix = None, False
        if self.v_mix:  # the first such layer leaves its values for the others
            mix = "values" in carry
            if not mix:
                carry["values"] = x.new_empty(x.shape[0], self.w.kv_heads * self.w.vdim)
            first = carry["values"]
        q = ops.attn_prep(proj, self.off_k, self.off_v, self.w, self.rope, meta.positions,
                          meta.slots, k, v, ring, v_first=first, mix=mix, **rows)
        gate = None if self.off_g is None else proj[:, self.off_g:self.off_g + self.w.heads]
        return q, gate

    def _decode(self, q, gate, dm, cache, out) -> None:
        ops.grouped_decode(q, cache[0], cache[1], self.w, gate, dm.block_tables, dm.context_lens,
                           dm.workspace.get(self.workspace_key(self.w)), out)

    def prefill(self, x, meta, cache, out=None, carry=None):
        step = meta.extra
        a = self._out(x, out)
        R, Tp, T = x.shape[0], meta.n_prefill, step.q_host[-1]
        q, gate = self._prep(x, meta, cache, carry, portions=step.portions, tiles=step.conv_tiles)

        def rows(lo, hi):
            return None if gate is None else gate[lo:hi]

        ops.grouped_prefill(q[:Tp], cache[0], cache[1], self.w, rows(0, Tp), step.grouped, a[:Tp])
        if T < Tp:
            a[T:Tp].zero_()
        if Tp < R:
            self._decode(q[Tp:], rows(Tp, R), meta.decode, cache, a[Tp:])
        return a

    def decode(self, x, meta, cache, out=None, carry=None):
        a = self._out(x, out)
        q, gate = self._prep(x, meta, cache, carry, row_state=meta.state)
        self._decode(q, gate, meta, cache, a)
        return a


class MemoryMixer(Mixer):
    """Retention or matrix memory: a matrix state per head with one decay."""

    def __init__(self, m: Retention | MatrixMemory, p: str, src, model):
        W, lin, f32 = model.cfg.hidden_size, model.lin, model.f32
        H, kd, vd = m.heads, m.heads * m.dim, m.heads * m.vdim
        gated = isinstance(m, MatrixMemory)
        sections = [src.take(p + x, n, W) for x, n in (("q", kd), ("k", kd), ("v", vd), ("g", vd))]
        if gated:
            sections += [src.take(p + x, H, W) for x in "if"]
        w, offs = fused_rows(sections)
        self.proj = lin(w)
        kw = dict(heads=H, dim=m.dim, vdim=m.vdim, eps=model.cfg.norm_eps, off_k=offs[1], off_v=offs[2],
                  off_g=offs[3])
        if gated:
            self.w = ops.MemoryWeights(
                **kw, act="sigmoid", q_scale=m.dim ** -0.5, off_i=offs[4], off_f=offs[5],
                i_bias=f32(src.take(p + "i.b", H)), f_bias=f32(src.take(p + "f.b", H)),
                cap=m.gate_cap, norm=f32(src.take(p + "norm", vd)))
        else:
            self.w = ops.MemoryWeights(
                **kw, act="silu", k_scale=m.dim ** -0.5, rot_dims=m.rot_dims,
                rope=model.rope(m.rot_base, m.rot_dims) if m.rot_dims else None,
                log_decay=f32(torch.tensor(m.decay, dtype=torch.float64).log()))
        self.width = vd
        self.o = lin(src.take(p + "o", W, vd))

    def operands(self):
        return [t for t in super().operands() if t is not self.w.rope]

    @staticmethod
    def _states(cache) -> tuple:
        return cache if isinstance(cache, tuple) else (cache, None, None)

    def prefill(self, x, meta, cache, out=None, carry=None):
        step = meta.extra
        a = self._out(x, out)
        R, Tp, T = x.shape[0], meta.n_prefill, step.q_host[-1]
        proj = ops.linear(x, self.proj)
        ops.memory_scan(proj, self.w, self._states(cache), step.portions, a, len(step.q_host) - 1)
        if T < Tp:
            a[T:Tp].zero_()
        if Tp < R:
            ops.memory_decode(proj[Tp:], self.w, self._states(cache), meta.positions[Tp:],
                              step.portions.row_state[Tp:], a[Tp:])
        return a

    def decode(self, x, meta, cache, out=None, carry=None):
        a = self._out(x, out)
        ops.memory_decode(ops.linear(x, self.proj), self.w, self._states(cache), meta.positions,
                          meta.state, a)
        return a


MIXERS = {Retention: MemoryMixer, MatrixMemory: MemoryMixer, LatentAttention: LatentMixer, ChannelDelta: DeltaMixer, TalkingAttention: TalkingMixer,
          GatedAverage: AverageMixer, GroupedAttention: GroupedMixer}
