"""Token mixers of per-layer mixed decoders on the serving engine's cache and slot state.

A mixer belongs to one run of a layer (a looped layer has one per pass): it names what it keeps -- KV pages
(``cache_shape``) and / or fp32 slot state (``state_widths``) -- and turns the layer's projection rows of a
batch (``hybrid_runner._Batch``) into the rows that the output projection reads.
"""
from __future__ import annotations

import dataclasses

import torch

from ..models.hybrid_config import (BiasedAttentionSpec, ChannelDeltaSpec, DiffAttentionSpec, GatedRecurrenceSpec,
                                    GeneralDeltaSpec, HeadDeltaSpec, LatentAttentionSpec, MatrixMemorySpec,
                                    PooledAttentionSpec, SideBySideSpec, SsdSpec, SumSpec, aligned_parts)
from ..ops import biased_attention as ba
from ..ops import delta_rule as dr
from ..ops import diff_attention as da
from ..ops import gated_scan as gs
from ..ops import latent_attention as la
from ..ops import matrix_memory as mm
from ..ops import moe
from ..ops import pooled_attention as pa
from ..ops import side_step as ss


class Mixer:
    """``run``: the layer run (names its state); ``linear``: the runner's projection; ``twin``: the mixer of an earlier
    pass over the same layer (shares what is derived from the weights). ``cache`` / ``index`` (the layer's first
    place in it) and ``state`` are set once the runner has made them. Mixers that a sum takes have ``weigh(mul)``."""

    def __init__(self, layer, cfg, run: int | str, linear, twin: Mixer | None = None):
        self.layer, self.run, self.linear = layer, run, linear
        self.cache = self.index = self.state = None

    def members(self) -> list:
        """The mixers that keep something: itself, or the ones it is made of."""
        return [self]

    def cache_shape(self):
        """(key heads, key size, value heads, value size) of the layer's pages, None without a cache."""
        return None

    def cache_shapes(self, page_size: int) -> list:
        """All pages of the layer, in the form of ``KVCache``'s ``layer_shapes``."""
        shape = self.cache_shape()
        return [] if shape is None else [shape]

    def state_widths(self) -> dict:
        return {}

    def buffers(self, rows: int, max_kv: int, dtype) -> dict:
        """Static workspaces of a decode bucket: name -> (elements, dtype); shared by the layers."""
        return {}

    def __call__(self, x, out, b):
        raise NotImplementedError


class DiffAttentionMixer(Mixer):
    def __init__(self, layer, cfg, run, linear, twin=None):
        super().__init__(layer, cfg, run, linear)
        mx = layer.spec.mixer
        self.sp = da.DiffHeads(mx.heads, mx.kv_heads, mx.dim, mx.vdim, mx.scale, layer.lam_value(), 1.0 - mx.diff,
                               cfg.norm_eps, mx.temp_coef, mx.temp_every)

    def cache_shape(self):
        mx = self.layer.spec.mixer
        return 2 * mx.kv_heads, mx.dim, mx.kv_heads, mx.vdim

    def buffers(self, rows, max_kv, dtype):
        _, _, w, c = da.rows_plan(self.sp, rows, max_kv, dtype)
        return {"ws": (w, torch.float32), "cnt": (c, torch.int32)}

    def __call__(self, qkv, out, b):
        sp, kc, vc, tbl = self.sp, self.cache.k[self.index], self.cache.v[self.index], self.cache.table
        a = (sp, qkv, kc, vc, tbl, b.pos, b.slots)
        if b.single:
            da.attend_rows(*a, out, b.max_kv, fused_append=True, ws=b.bufs.get("ws"), cnt=b.bufs.get("cnt"))
            return
        da.append(*a)
        if out.is_cuda and da.tiles_ok(sp, out.dtype, self.cache.page_size, out.stride(0)):
            if b.tiles is not None:
                da.attend_tiles(*a, out, b.tiles)
            if b.row_of is not None:
                da.attend_rows(*a, out, b.row_kv, fused_append=False, row_of=b.row_of)
        else:
            da.attend_rows(*a, out, b.max_kv, fused_append=False)


class GatedRecurrenceMixer(Mixer):
    def state_widths(self):
        return {f"scan{self.run}": (1, self.layer.spec.mixer.width)}

    def __call__(self, zxg, out, b):
        L, st = self.layer, self.state[f"scan{self.run}"][0]
        if b.single:
            gs.gated_step(zxg, L.b_z, L.b_x, st, out, b.pos, b.slots)
        else:
            gs.gated_scan(zxg, L.b_z, L.b_x, st, out, b.chunks, b.multi)


class LatentAttentionMixer(Mixer):
    def __init__(self, layer, cfg, run, linear, twin=None):
        super().__init__(layer, cfg, run, linear)
        mx, L = layer.spec.mixer, layer
        self.sp = sp = la.LatentHeads(mx.heads, mx.dim, mx.rot_dim, mx.vdim, mx.q_rank, mx.kv_rank, mx.scale,
                                      cfg.norm_eps, mx.rot_base, mx.rot_dims, (mx.parts["dq"][0], mx.parts["dkv"][0]))
        nk = sp.heads * sp.dim
        self.wt = twin.wt if twin is not None else la.LatentWeights(L.q_norm, L.kv_norm, L.sink,
                                   L.ukv[:nk].view(sp.heads, sp.dim, sp.kv_rank).transpose(1, 2).contiguous(),
                                   L.ukv[nk:].view(sp.heads, sp.vdim, sp.kv_rank), sp.frequencies().to(L.ukv.device))

    def cache_shape(self):
        return 1, self.sp.row, 0, 0

    def buffers(self, rows, max_kv, dtype):
        return {"part": (la.rows_plan(self.sp, rows, max_kv)[2], torch.float32)}

    def __call__(self, x, out, b):
        sp, wt, pages, tbl = self.sp, self.wt, self.cache.k[self.index], self.cache.table
        a = (pages, tbl, b.pos, b.slots)
        q = self.linear(la.latent_append(sp, wt, x, *a), self.layer.uq)
        pr = b.prompts
        if pr is None or not pr.tiles.shape[0] or not (out.is_cuda and la.tiles_ok(sp, out.dtype, out.stride(0))):
            la.attend_rows(sp, wt, q, *a, out, b.max_kv, part=b.bufs.get("part"))
            return
        la.attend_prompts(sp, wt, q, *a, out, self.layer.ukv, pr, self.linear)
        if pr.rows.shape[0]:
            la.attend_rows(sp, wt, q, *a, out, pr.rows_kv, row_of=pr.rows)


class DeltaRuleMixer(Mixer):
    def __init__(self, layer, cfg, run, linear, twin=None):
        super().__init__(layer, cfg, run, linear)
        mx, L = layer.spec.mixer, layer
        at = lambda *names: tuple(mx.parts[n][0] for n in names)  # noqa: E731
        if isinstance(mx, GeneralDeltaSpec):
            self.sp = dr.DeltaHeads(True, mx.heads, mx.heads, mx.dim, mx.dim, at("r", "k", "v", "a", "g", "w1"),
                                    mx.rank_w, cfg.norm_eps)
            self.wt = dr.DeltaWeights(L.w2, L.w0, L.a_bias, L.gain)
        elif isinstance(mx, HeadDeltaSpec):
            self.sp = dr.DeltaHeads(False, mx.heads, mx.kv_heads, mx.dim, mx.vdim, at("q", "k", "v", "b", "g", "a"), 0,
                                    cfg.norm_eps, mx.taps, form="head")
            self.wt = dr.DeltaWeights(None, L.dt_bias, L.a_log, L.gain, conv=L.conv)
        elif isinstance(mx, SsdSpec):
            self.sp = dr.DeltaHeads(False, mx.heads, mx.groups, mx.state, mx.vdim, at("C", "B", "x", "dt", "z", "dt"), 0,
                                    cfg.norm_eps, mx.taps, form="ssd", norm_groups=mx.norm_groups)
            self.wt = dr.DeltaWeights(None, L.dt_bias, L.a_log, L.gain, conv=L.conv, conv_b=L.conv_b, skip=L.skip)
        else:
            self.sp = dr.DeltaHeads(False, mx.heads, mx.kv_heads, mx.dim, mx.vdim, at("q", "k", "v", "b", "g1", "a1"),
                                    mx.rank_w, cfg.norm_eps, mx.taps, mx.rank_g)
            self.wt = dr.DeltaWeights(L.a2, L.dt_bias, L.a_log, L.gain, L.g2, L.conv)

    def state_widths(self):
        w = {f"delta{self.run}": (1, self.sp.state_width)}
        if not self.sp.general:
            w[f"ring{self.run}"] = (1, self.sp.taps * self.sp.conv_channels)
        return w

    def __call__(self, x, out, b):
        sp, wt = self.sp, self.wt
        S = self.state[f"delta{self.run}"][0]
        ring = None if sp.general else self.state[f"ring{self.run}"][0]
        if b.single:
            dr.delta_step(sp, wt, x, S, ring, b.pos, b.slots, out)
            return
        if sp.kind >= 2:
            dr.delta_portions(sp, wt, x, S, ring, b.portions, out)
            return
        tanh = lambda t: moe.act_rows(t, torch.empty_like(t, memory_format=torch.contiguous_format), False, act="tanh")  # noqa: E731
        inner, gate = dr.low_rank_inner(sp, x, tanh)
        dr.delta_portions(sp, wt, x, S, ring, b.portions, out, self.linear(inner, wt.lo_w),
                          None if gate is None else self.linear(gate, wt.lo_g))


class BiasedAttentionMixer(Mixer):
    def __init__(self, layer, cfg, run, linear, twin=None):
        super().__init__(layer, cfg, run, linear)
        mx, L = layer.spec.mixer, layer
        self.sp = ba.BiasedHeads(mx.heads, mx.kv_heads, mx.dim, mx.vdim, mx.scale, cfg.norm_eps,
                                 tuple(mx.parts[n][0] for n in "qkvg"))
        self.wt = twin.wt if twin is not None else ba.BiasedWeights(L.q_norm, L.k_norm, ba.bias_by_distance(L.rel, mx.bias_max),
                                                                    L.sink.float())

    def cache_shape(self):
        mx = self.layer.spec.mixer
        return mx.kv_heads, mx.dim, mx.kv_heads, mx.vdim

    def buffers(self, rows, max_kv, dtype):
        _, _, w, c = ba.rows_plan(self.sp, rows, max_kv)
        return {"ws": (w, torch.float32), "cnt": (c, torch.int32)}

    def __call__(self, x, out, b):
        a = (self.sp, self.wt, x, self.cache.k[self.index], self.cache.v[self.index], self.cache.table, b.pos, b.slots)
        if b.single:
            ba.attend_rows(*a, out, b.max_kv, fused_append=True, ws=b.bufs.get("ws"), cnt=b.bufs.get("cnt"))
            return
        ba.append(*a)
        if out.is_cuda and ba.tiles_ok(self.sp, out.dtype, self.cache.page_size, x.stride(0), out.stride(0)):
            if b.tiles is not None:
                ba.attend_tiles(*a, out, b.tiles)
            if b.row_of is not None:
                ba.attend_rows(*a, out, b.row_kv, fused_append=False, row_of=b.row_of)
        else:
            ba.attend_rows(*a, out, b.max_kv, fused_append=False)


class PooledAttentionMixer(Mixer):
    """The block means lie beside the tokens' keys and values in the same pages: a second entry of the cache."""

    def __init__(self, layer, cfg, run, linear, twin=None):
        super().__init__(layer, cfg, run, linear)
        mx, L = layer.spec.mixer, layer
        self.sp = pa.PooledHeads(mx.heads, mx.kv_heads, mx.dim, mx.vdim, mx.scale, cfg.norm_eps,
                                 tuple(mx.parts[n][0] for n in "qkv"), mx.window, mx.pool, mx.rot_dims)
        self.wt = twin.wt if twin is not None else pa.PooledWeights(
            L.q_norm, L.k_norm, L.sink.float(), pa.rotary_frequencies(mx.rot_dims, mx.rot_base, mx.rot_scaling).to(L.sink.device))

    def weigh(self, mul: float):
        self.sp = dataclasses.replace(self.sp, mul=mul)

    def cache_shape(self):
        mx = self.layer.spec.mixer
        return mx.kv_heads, mx.dim, mx.kv_heads, mx.vdim

    def cache_shapes(self, page_size):
        shape = self.cache_shape()
        return [shape, (*shape, pa.block_rows(page_size, self.sp.pool))]

    def buffers(self, rows, max_kv, dtype):
        _, _, w, c = pa.rows_plan(self.sp, rows, self.sp.visible(max_kv))
        return {"ws": (w, torch.float32), "cnt": (c, torch.int32)}

    def pages(self):
        c, i = self.cache, self.index
        return pa.PooledCache(c.k[i], c.v[i], c.k[i + 1], c.v[i + 1], c.table)

    def __call__(self, x, out, b):
        a = (self.sp, self.wt, x, self.pages(), b.pos, b.slots)
        if b.single:
            pa.attend_rows(*a, out, b.max_kv, fused=True, ws=b.bufs.get("ws"), cnt=b.bufs.get("cnt"))
            return
        pa.prepare(*a)
        if out.is_cuda and pa.tiles_ok(self.sp, out.dtype, self.cache.page_size, x.stride(0), out.stride(0)):
            if b.tiles is not None:
                pa.attend_tiles(*a, out, b.tiles)
            if b.row_of is not None:
                pa.attend_rows(*a, out, b.row_kv, fused=False, row_of=b.row_of)
        else:
            pa.attend_rows(*a, out, b.max_kv, fused=False)


class MatrixMemoryMixer(Mixer):
    def __init__(self, layer, cfg, run, linear, twin=None):
        super().__init__(layer, cfg, run, linear)
        mx, L = layer.spec.mixer, layer
        self.sp = mm.MemoryHeads(mx.heads, mx.dim, mx.vdim, tuple(mx.parts[n][0] for n in "qkvgif"), mx.gate_cap, cfg.norm_eps)
        self.wt = mm.MemoryWeights(L.i_bias, L.f_bias, L.gain)

    def weigh(self, mul: float):
        self.sp = dataclasses.replace(self.sp, mul=mul)

    def state_widths(self):
        sp, r = self.sp, self.run
        return {f"mem{r}": (1, sp.heads * sp.dim * sp.vdim), f"memn{r}": (1, sp.heads * sp.dim), f"memm{r}": (1, sp.heads)}

    def memory(self):
        return mm.MemoryState(*(self.state[f"{k}{self.run}"][0] for k in ("mem", "memn", "memm")))

    def __call__(self, x, out, b):
        st = self.memory()
        if b.single:
            mm.memory_step(self.sp, self.wt, x, st, b.pos, b.slots, out)
        else:
            mm.memory_portions(self.sp, self.wt, x, st, b.portions, out)


class SideBySideMixer(Mixer):
    """Two mixers over column blocks of the projection rows, into column blocks of the output rows."""

    def __init__(self, layer, cfg, run, linear, twin=None):
        super().__init__(layer, cfg, run, linear)
        self.sides = [make_mixer(m, cfg, f"{run}.{k}", linear, twin and twin.sides[k]) for k, m in enumerate((layer.left, layer.right))]
        mx = layer.spec.mixer
        self.cols = (slice(0, mx.left.in_rows), slice(mx.in_rows - mx.right.in_rows, mx.in_rows))
        parts, self.out_width = aligned_parts({"left": mx.left.out_cols, "right": mx.right.out_cols})
        self.outs = tuple(slice(o, o + n) for o, n in parts.values())

    def members(self):
        return [m for s in self.sides for m in s.members()]

    def __call__(self, x, out, b):
        for m, c, o in zip(self.sides, self.cols, self.outs):
            m(x[:, c], out[:, o], b)


class SumMixer(SideBySideMixer):
    """... whose rows carry the sides' weights, so that one output projection sums them."""

    def __init__(self, layer, cfg, run, linear, twin=None):
        super().__init__(layer, cfg, run, linear, twin)
        mx = layer.spec.mixer
        for m, mul in zip(self.sides, (mx.left_mul, mx.right_mul)):
            m.weigh(mul)
        self.pooled_memory = [type(m) for m in self.sides] == [PooledAttentionMixer, MatrixMemoryMixer]

    def __call__(self, x, out, b):
        if b.single and self.pooled_memory:  # a decode step of both in one launch
            (l, r), (xl, xr), (ol, orr) = self.sides, (x[:, c] for c in self.cols), (out[:, o] for o in self.outs)
            if ss.step_ok(l.sp, r.sp, xl):
                ss.step((l.sp, l.wt, xl, l.pages(), ol), (r.sp, r.wt, xr, r.memory(), orr), b.pos, b.slots, b.max_kv,
                        b.bufs.get("ws"), b.bufs.get("cnt"))
                return
        super().__call__(x, out, b)


MIXERS = {DiffAttentionSpec: DiffAttentionMixer, GatedRecurrenceSpec: GatedRecurrenceMixer,
          LatentAttentionSpec: LatentAttentionMixer, GeneralDeltaSpec: DeltaRuleMixer, ChannelDeltaSpec: DeltaRuleMixer,
          HeadDeltaSpec: DeltaRuleMixer, SsdSpec: DeltaRuleMixer, BiasedAttentionSpec: BiasedAttentionMixer,
          SideBySideSpec: SideBySideMixer, PooledAttentionSpec: PooledAttentionMixer, MatrixMemorySpec: MatrixMemoryMixer,
          SumSpec: SumMixer}


def make_mixer(layer, cfg, run: int | str, linear, twin: Mixer | None = None) -> Mixer:
    return MIXERS[type(layer.spec.mixer)](layer, cfg, run, linear, twin)


__all__ = ["Mixer", "MIXERS", "make_mixer"]
