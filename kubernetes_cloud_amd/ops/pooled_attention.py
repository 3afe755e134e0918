"""Sliding-window attention over the paged cache that sees what lies before its window as block means
(``csrc/kernels/pooled_attn.hip``).

    q <- R(pos) N(q),  k <- R(pos) N(k)              N: RMS norm over all heads at once, with a gain
    w_j = exp(q . k_j * scale),  o = mul * sum_j w_j v_j / (exp(sink_h) + sum_j w_j)

A query at pos sees the tokens (pos - window, pos] and, as one key and value each, the means of the whole blocks of
``pool`` tokens that end at or before pos - window. R rotates the first ``rot`` dims of a head in pairs (i, i + rot / 2).
Query heads share key / value heads in groups; q / k / v are column blocks of one buffer.

Cache: K pages [pages, G, PS, dim] (normed, rotated keys), V pages [pages, G, PS, vdim], and beside them in the same pages
the means of the blocks that end there, [pages, G, per, dim] / [.., vdim]: block b in row (end % PS) // pool. So a
block lives and is shared, copied and given back with the page of its last token.
"""
from __future__ import annotations

import ctypes
import dataclasses
import math

import torch

from . import _lib
from . import biased_attention as ba
from .decode import gather_kv
from .rms_shift import native_dt

SPLIT_TARGET, SPLIT_MIN = 1024, 96


@dataclasses.dataclass(frozen=True)
class PooledHeads:
    """Sizes and constants of one layer's attention. ``at``: first columns of q, k and v; ``rot``: rotated dims."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    eps: float
    at: tuple
    window: int
    pool: int
    rot: int = 0
    mul: float = 1.0

    def visible(self, n: int) -> int:
        """Keys (tokens and block means) that the last of ``n`` tokens sees."""
        return min(n, self.window) + max(0, n - self.window) // self.pool


@dataclasses.dataclass(frozen=True)
class PooledWeights:
    """Gains of the norms [H dim], [G dim]; ``sink`` fp32 [H]; ``freq`` fp32 [rot / 2], radians per position."""
    q_norm: torch.Tensor
    k_norm: torch.Tensor
    sink: torch.Tensor
    freq: torch.Tensor


@dataclasses.dataclass(frozen=True)
class PooledCache:
    """Pages of the tokens' keys and values and of the block means, and the slots' page table."""
    k: torch.Tensor
    v: torch.Tensor
    kb: torch.Tensor
    vb: torch.Tensor
    table: torch.Tensor


def block_rows(page_size: int, pool: int) -> int:
    """Block means a page can hold."""
    return -(-page_size // pool)


def rotary_frequencies(dims: int, base: float, scaling: tuple | None = None) -> torch.Tensor:
    """Radians per position of each pair, fp32 [dims / 2]: base^(-2 i / dims). ``scaling`` (factor, low, high, original)
    slows the pairs whose wavelength exceeds original / low by ``factor``, keeps those below original / high, and
    mixes both between (the Llama 3.1 rule)."""
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if scaling is not None:
            factor, low, high, original = scaling
            turns = original * f / (2 * math.pi)  # within the original length
            if turns < low:
                f /= factor
            elif turns <= high:
                s = (turns - low) / (high - low)
                f = (1 - s) * f / factor + s * f
        out.append(f)
    return torch.tensor(out, dtype=torch.float64).float()


def rows_plan(sp: PooledHeads, rows: int, max_kv: int) -> tuple[int, int, int, int]:
    """``biased_attention.rows_plan`` over the keys that are seen: about four workgroups a CU, of 96 keys or more
    (a window bounds the rows' keys, so they differ little and splits of one size fill the chip evenly)."""
    return ba.rows_plan(sp, rows, max_kv, SPLIT_TARGET, SPLIT_MIN)


def tiles_ok(sp: PooledHeads, dtype, page_size: int, ld: int, ldo: int) -> bool:
    """Shapes the matrix-core kernel takes (others run the rows kernel)."""
    return ba.tiles_ok(sp, dtype, page_size, ld, ldo)


def _args(sp: PooledHeads, wt: PooledWeights, x, c: PooledCache, pos, slots, out=None) -> ba._Args:
    G, D, E, PS = sp.kv_heads, sp.dim, sp.vdim, c.k.shape[2]
    per, pages = block_rows(PS, sp.pool), c.k.shape[0]
    assert sp.window >= 1 and 1 <= sp.pool <= 1 << 20 and PS <= 1024 and sp.rot % 2 == 0 and 0 <= sp.rot <= D
    assert c.kb.is_contiguous() and c.kb.shape == (pages, G, per, D) and c.vb.is_contiguous() and c.vb.shape == (pages, G, per, E)
    assert all(t.is_contiguous() and t.numel() == n * D and t.dtype == x.dtype
               for t, n in ((wt.q_norm, sp.heads), (wt.k_norm, G)))
    assert wt.freq.is_contiguous() and wt.freq.dtype == torch.float32 and wt.freq.numel() == sp.rot // 2
    if _lib.require().kca_pooled_attn_abi() != ctypes.sizeof(ba._Args):
        raise RuntimeError("kca_pooled_attn descriptor: C and ctypes sizes differ")
    core = ba.BiasedHeads(sp.heads, G, D, E, sp.scale, sp.eps, (*sp.at, -1))
    a = ba._args(core, ba.BiasedWeights(sink=wt.sink), x, c.k, c.v, c.table, pos, slots, out)
    a.qn, a.kn, a.freq, a.rot, a.mul = wt.q_norm.data_ptr(), wt.k_norm.data_ptr(), wt.freq.data_ptr(), sp.rot, sp.mul
    a.window, a.pool, a.per, a.pool_mul = sp.window, sp.pool, per, -(-(1 << 20) // sp.pool)
    a.kb, a.vb, a.kb_sp, a.vb_sp = c.kb.data_ptr(), c.vb.data_ptr(), c.kb.stride(0), c.vb.stride(0)
    return a


def prepare(sp: PooledHeads, wt: PooledWeights, x, c: PooledCache, pos, slots):
    """Norms and rotation of every row of ``x``: queries in place, keys and values into their pages, and the means of
    the blocks these rows complete."""
    code = native_dt(x, c.k, c.v, c.kb, c.vb)
    if code is None:
        return _prepare_reference(sp, wt, x, c, pos, slots)
    ba._call("kca_pooled_prep", _args(sp, wt, x, c, pos, slots), code, x.shape[0])


def attend_rows(sp: PooledHeads, wt: PooledWeights, x, c: PooledCache, pos, slots, out, max_len: int, *, fused: bool,
                row_of: torch.Tensor | None = None, ws: torch.Tensor | None = None, cnt: torch.Tensor | None = None):
    """One query token per row (sequences of up to ``max_len`` tokens). ``fused``: the rows come as projected, one
    token per sequence, and are prepared on the way; else ``prepare`` has run. ``row_of``: only these rows."""
    code = native_dt(x, c.k, c.v, out)
    if code is None:
        if fused:
            _prepare_reference(sp, wt, x, c, pos, slots)
        return _reference(sp, wt, x, c, pos, slots, out, range(x.shape[0]) if row_of is None else row_of.tolist())
    a, n, wsn, cn, kv, keep = rows_args(sp, wt, x, c, pos, slots, out, max_len, fused, row_of, ws, cnt)
    ba._call("kca_pooled_rows", a, code, n, wsn, cn, kv)
    del keep
    return out


def rows_args(sp, wt, x, c, pos, slots, out, max_len, fused, row_of, ws, cnt):
    """The rows kernel's descriptor -> (descriptor, rows, workspace floats, counters, most keys, what must stay alive until
    the launch)."""
    n = x.shape[0] if row_of is None else row_of.shape[0]
    kv = sp.visible(max_len)
    splits, chunk, wsf, blocks = rows_plan(sp, n, kv)
    if splits > 1:
        if ws is None or ws.numel() < wsf:
            ws = torch.empty(wsf, device=x.device, dtype=torch.float32)
        if cnt is None or cnt.numel() < blocks:
            cnt = torch.zeros(blocks, device=x.device, dtype=torch.int32)
    a = _args(sp, wt, x, c, pos, slots, out)
    a.append, a.nsplit, a.chunk, a.row_of = int(fused), splits, chunk, _lib.ptr(row_of)
    a.ws, a.cnt = _lib.ptr(ws), _lib.ptr(cnt)
    assert row_of is None or row_of.dtype == torch.int32
    return a, n, ws.numel() if ws is not None else 0, cnt.numel() if cnt is not None else 0, kv, (ws, cnt)


def attend_tiles(sp: PooledHeads, wt: PooledWeights, x, c: PooledCache, pos, slots, out, tiles: torch.Tensor):
    """Prepared prompt portions (``diff_attention.plan_tiles``) on the matrix cores."""
    assert native_dt(x, c.k, c.v, out) == 1 and tiles.dtype == torch.int32 and tiles.is_contiguous()
    a = _args(sp, wt, x, c, pos, slots, out)
    a.tiles = tiles.data_ptr()
    ba._call("kca_pooled_tiles", a, tiles.shape[0])
    return out


def _block_at(c: PooledCache, pool: int, slot: int, b: int) -> tuple[int, int]:
    """(page, row) of block ``b`` of a slot."""
    page, row = divmod(b * pool + pool - 1, c.k.shape[2])
    return int(c.table[slot, page]), row // pool


def _prepare_reference(sp, wt, x, c, pos, slots):
    T, (H, G, D, E), PS = x.shape[0], (sp.heads, sp.kv_heads, sp.dim, sp.vdim), c.k.shape[2]
    pos, slots = pos.long()[:T], slots.long()[:T]
    ang = pos[:, None].float() * wt.freq
    cos, sin, n = torch.cos(ang)[:, None], torch.sin(ang)[:, None], sp.rot // 2

    def heads(o, count, gain):
        u = x[:, o:o + count * D].float()
        u = (u * torch.rsqrt((u * u).mean(-1, keepdim=True) + sp.eps) * gain.float()).view(T, count, D)
        a, b = u[..., :n], u[..., n:2 * n]
        return torch.cat([a * cos - b * sin, b * cos + a * sin, u[..., 2 * n:]], -1).to(x.dtype)

    q, k = heads(sp.at[0], H, wt.q_norm), heads(sp.at[1], G, wt.k_norm)
    x[:, sp.at[0]:sp.at[0] + H * D] = q.reshape(T, H * D)
    pg = c.table.long()[slots, pos // PS]
    c.k[pg, :, pos % PS] = k
    c.v[pg, :, pos % PS] = x[:, sp.at[2]:sp.at[2] + G * E].reshape(T, G, E)
    for p, s in zip(pos.tolist(), slots.tolist()):
        if (p + 1) % sp.pool == 0:
            page, row = _block_at(c, sp.pool, s, p // sp.pool)
            for src, dst in ((c.k, c.kb), (c.v, c.vb)):
                dst[page, :, row] = gather_kv(src, s, p + 1, c.table)[:, p + 1 - sp.pool:].float().mean(1).to(dst.dtype)


def _reference(sp, wt, x, c, pos, slots, out, rows):
    H, G, D, E = sp.heads, sp.kv_heads, sp.dim, sp.vdim
    for t in rows:
        p, s = int(pos[t]), int(slots[t])
        lo, nb = max(0, p - sp.window + 1), max(0, p - sp.window + 1) // sp.pool
        at = [_block_at(c, sp.pool, s, b) for b in range(nb)]
        kv = []
        for pages, means in ((c.k, c.kb), (c.v, c.vb)):
            seen = [gather_kv(pages, s, p + 1, c.table)[:, lo:].float()]
            if at:
                seen.insert(0, torch.stack([means[a, :, r] for a, r in at], 1).float())
            kv.append(torch.cat(seen, 1))  # [G, n, size]
        q = x[t, sp.at[0]:sp.at[0] + H * D].float().view(G, H // G, D)
        w = (torch.matmul(q, kv[0].transpose(-1, -2)) * sp.scale).reshape(H, -1)
        w = torch.softmax(torch.cat([w, wt.sink[:, None]], 1), -1)[:, :-1].view(G, H // G, -1)
        out[t] = (torch.matmul(w, kv[1]).reshape(H * E) * sp.mul).to(out.dtype)
    return out


__all__ = ["PooledHeads", "PooledWeights", "PooledCache", "block_rows", "rotary_frequencies", "prepare", "attend_rows",
           "attend_tiles", "rows_plan", "tiles_ok"]
