"""Latent attention over the paged cache (``csrc/kernels/latent_attn.h``).

Few query tokens attend over the latents themselves (``attend_rows``); prompt portions expand their context's
keys and values once and run as tiles of queries (``attend_prompts``). bf16 takes the matrix-core kernels of
``latent_mfma.hip`` wherever the sizes allow, everything else ``latent_attn.hip``.

The cache holds one row per token, [c (kv_rank, normed) | r (rot_dim, rotated key part)], shared by all heads:
pages [n, 1, PS, kv_rank + rot_dim]. A head's key is [W_uk c | r], its value W_uv c, so a score is
(W_uk^T q) . c + rot(q) . r and an output W_uv (sum_j weight_j c_j); exp(sink) joins the softmax's denominator.
"""
from __future__ import annotations

import ctypes
import dataclasses

import numpy as np
import torch

from . import _lib
from .decode import gather_kv
from .rms_shift import native_dt


_P, _LL, _I, _F = ctypes.c_void_p, ctypes.c_longlong, ctypes.c_int, ctypes.c_float


class _Args(ctypes.Structure):
    _fields_ = [("x", _P), ("ld", _LL), *[(n, _I) for n in ("o_q", "o_kv", "H", "D", "R", "E", "C", "Q", "nr")],
                ("gq", _P), ("gk", _P), ("eps", _F), ("scale", _F), ("cq", _P), ("kc", _P), ("k_sp", _LL),
                ("table", _P), ("tstride", _I), ("shift", _I), ("pos", _P), ("slot", _P), ("freq", _P), ("q", _P),
                ("qa", _P), ("sink", _P), ("part", _P), ("nsplit", _I), ("chunk", _I), ("row_of", _P), ("wuv", _P),
                ("out", _P), ("ldo", _LL), ("kv", _P), ("ldkv", _LL), ("kr", _P), ("tiles", _P)]


TILE = 128        # query rows of a prompt tile
PROMPT_MIN = 32   # shorter portions run row by row
MAX_SPLITS = 256


@dataclasses.dataclass(frozen=True)
class LatentHeads:
    """Sizes and constants of one layer. ``at``: first columns of the query latent and of [latent | rotated part]
    in the projection rows."""
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    eps: float
    rot_base: float
    rot_dims: int
    at: tuple

    @property
    def row(self) -> int:
        return self.kv_rank + self.rot_dim

    def frequencies(self) -> torch.Tensor:
        """Radians per position of every rotated pair (rounded once to fp32)."""
        i = torch.arange(self.rot_dims // 2, dtype=torch.float64)
        return (self.rot_base ** (-2 * i / max(1, self.rot_dims))).float()


@dataclasses.dataclass(frozen=True)
class LatentWeights:
    """``wuk_t`` [H, kv_rank, dim] (W_uk transposed per head), ``wuv`` [H, vdim, kv_rank]."""
    q_norm: torch.Tensor
    kv_norm: torch.Tensor
    sink: torch.Tensor
    wuk_t: torch.Tensor
    wuv: torch.Tensor
    freq: torch.Tensor


def rotate(sp: LatentHeads, wt: LatentWeights, x, pos):
    """Reference rotation of the last axis of x [T, ..., rot_dim] (fp32)."""
    n = sp.rot_dims
    a = pos.float()[:, None] * wt.freq
    c, s = torch.cos(a), torch.sin(a)
    while c.dim() < x.dim():
        c, s = c[:, None], s[:, None]
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    y = torch.stack([u * c - v * s, v * c + u * s], -1).flatten(-2)
    return torch.cat([y, x[..., n:]], -1)


def _base(sp: LatentHeads, wt: LatentWeights, pages, table, pos, slots, T) -> _Args:
    PS = pages.shape[2]
    assert pages.is_contiguous() and pages.shape[1:] == (1, PS, sp.row) and PS >= 16 and PS & (PS - 1) == 0
    assert table.dtype == torch.int32 and table.is_contiguous() and wt.freq.dtype == torch.float32
    assert wt.freq.numel() == sp.rot_dims // 2
    assert pos.dtype == torch.int32 and slots.dtype == torch.int32 and pos.shape[0] >= T and slots.shape[0] >= T
    if _lib.require().kca_latent_abi() != ctypes.sizeof(_Args):
        raise RuntimeError("kca_latent descriptor: C and ctypes sizes differ")
    a = _Args()
    a.H, a.D, a.R, a.E, a.C, a.Q, a.nr = (sp.heads, sp.dim, sp.rot_dim, sp.vdim, sp.kv_rank, sp.q_rank, sp.rot_dims)
    a.eps, a.scale = sp.eps, sp.scale
    a.kc, a.k_sp = pages.data_ptr(), pages.stride(0)
    a.table, a.tstride, a.shift = table.data_ptr(), table.stride(0), PS.bit_length() - 1
    a.pos, a.slot, a.freq = pos.data_ptr(), slots.data_ptr(), wt.freq.data_ptr()
    return a


def _call(name, a, *args, other: bool = False) -> bool:
    """``other``: status 10 (sizes for another kernel) returns False instead of raising."""
    fn = getattr(_lib.require(), name)
    fn.argtypes = [ctypes.c_void_p] + [ctypes.c_int] * len(args) + [ctypes.c_void_p]
    fn.restype = ctypes.c_int
    rc = fn(ctypes.addressof(a), *args, _lib.stream())
    if rc == 10 and other:
        return False
    if rc != 0:
        raise RuntimeError(f"{name} returned status {rc} (unsupported shape/arguments)")
    _lib.LAUNCHES[0] += 1
    if _lib.SYNC_LAUNCH:
        torch.cuda.synchronize()
    return True


def latent_append(sp: LatentHeads, wt: LatentWeights, x, pages, table, pos, slots) -> torch.Tensor:
    """Cache rows of every token of the projection rows ``x`` into their pages. -> normed query latents [T, Q]."""
    T = x.shape[0]
    code = native_dt(x, pages, wt.q_norm, wt.kv_norm)
    assert x.stride(1) == 1 and sp.at[0] + sp.q_rank <= x.shape[1] and sp.at[1] + sp.row <= x.shape[1]
    if code is None:
        rms = lambda y: y * torch.rsqrt((y * y).mean(-1, keepdim=True) + sp.eps)  # noqa: E731
        xq = x[:, sp.at[0]:sp.at[0] + sp.q_rank].float()
        xk = x[:, sp.at[1]:sp.at[1] + sp.row].float()
        c = rms(xk[:, :sp.kv_rank]) * wt.kv_norm.float()
        r = rotate(sp, wt, xk[:, sp.kv_rank:], pos[:T])
        PS = pages.shape[2]
        pages[table.long()[slots.long()[:T], pos.long()[:T] // PS], 0, pos.long()[:T] % PS] = torch.cat([c, r], 1).to(x.dtype)
        return (rms(xq) * wt.q_norm.float()).to(x.dtype)
    cq = torch.empty(T, sp.q_rank, device=x.device, dtype=x.dtype)
    a = _base(sp, wt, pages, table, pos, slots, T)
    a.x, a.ld, a.o_q, a.o_kv = x.data_ptr(), x.stride(0), *sp.at
    a.gq, a.gk, a.cq = wt.q_norm.data_ptr(), wt.kv_norm.data_ptr(), cq.data_ptr()
    assert wt.q_norm.numel() == sp.q_rank and wt.kv_norm.numel() == sp.kv_rank
    _call("kca_latent_prep", a, code, T)
    return cq


def rows_plan(sp: LatentHeads, rows: int, max_kv: int) -> tuple[int, int, int]:
    """(splits, keys per split, partial floats)."""
    want = -(-512 // (rows * -(-sp.heads // 32)))  # two workgroups a CU, 64 keys each at least
    chunk = max_kv if rows * sp.heads >= 4096 else max(64, -(-max_kv // want))
    chunk = -(-max(chunk, -(-max_kv // MAX_SPLITS)) // 64) * 64
    n = -(-max_kv // chunk)
    return n, chunk, rows * sp.heads * n * (sp.kv_rank + 4)


def attend_rows(sp: LatentHeads, wt: LatentWeights, q, pages, table, pos, slots, out, max_kv: int, *,
                row_of: torch.Tensor | None = None, part: torch.Tensor | None = None):
    """One query token per row (``row_of``: only these rows) over its keys [0, pos], which the pages hold.
    ``q`` [T, H (dim + rot_dim)] unrotated."""
    code = native_dt(q, pages, wt.wuk_t, wt.wuv, wt.sink, out)
    T, H, D = q.shape[0], sp.heads, sp.dim
    assert q.is_contiguous() and q.shape[1] == H * (D + sp.rot_dim) and out.stride(1) == 1 and out.shape == (T, H * sp.vdim)
    n = T if row_of is None else row_of.shape[0]
    if code is None:
        return _reference(sp, wt, q, pages, table, pos, slots, out, range(T) if row_of is None else row_of.tolist())
    assert wt.wuk_t.is_contiguous() and wt.wuk_t.shape == (H, sp.kv_rank, D) and wt.sink.numel() == H
    assert wt.wuv.is_contiguous() and wt.wuv.shape == (H, sp.vdim, sp.kv_rank)
    assert row_of is None or row_of.dtype == torch.int32
    splits, chunk, need = rows_plan(sp, n, max_kv)
    if part is None or part.numel() < need:
        part = torch.empty(need, device=q.device, dtype=torch.float32)
    qa = torch.empty(n, H * sp.kv_rank, device=q.device, dtype=q.dtype)
    head_mm(q, D + sp.rot_dim, wt.wuk_t, qa, row_of)
    a = _base(sp, wt, pages, table, pos, slots, T)
    a.q, a.qa, a.part, a.nsplit, a.chunk = q.data_ptr(), qa.data_ptr(), part.data_ptr(), splits, chunk
    a.row_of, a.sink, a.wuv = _lib.ptr(row_of), wt.sink.data_ptr(), wt.wuv.data_ptr()
    a.out, a.ldo = out.data_ptr(), out.stride(0)
    if code != 1 or not _call("kca_latent_rows_mfma", a, n, int(max_kv), other=True):
        _call("kca_latent_rows", a, code, n, int(max_kv))
    if code != 1 or not _call("kca_latent_merge_mfma", a, n, other=True):
        _call("kca_latent_merge", a, code, n)
    return out


@dataclasses.dataclass
class Prompts:
    """Device arrays of the portions that run as tiles (``plan_prompts``): ``tiles`` [n, 4] first row, rows,
    position of the first row, context row of position 0 (longest key ranges first); ``ctx`` [m, 3] first context
    row, length, slot; ``rows`` the token rows of all other entries."""
    tiles: torch.Tensor
    ctx: torch.Tensor
    rows: torch.Tensor
    n_ctx: int      # context rows
    max_ctx: int    # longest context
    rows_kv: int    # keys the longest of the other rows sees


def plan_prompts(entries, min_rows: int = PROMPT_MIN) -> tuple[dict, dict]:
    """[(first row, rows, position, slot)] -> (host arrays, host numbers) of ``Prompts``."""
    tiles, ctx, rows, at, kv = [], [], [], 0, 0
    for r0, n, p0, slot in entries:
        if n < min_rows:
            rows += range(r0, r0 + n)
            kv = max(kv, p0 + n)
            continue
        ctx.append((at, p0 + n, slot))
        tiles += [(r0 + i, min(TILE, n - i), p0 + i, at) for i in range(0, n, TILE)]
        at += p0 + n
    tiles.sort(key=lambda t: -(t[2] + t[1]))
    arr = {"tiles": np.asarray(tiles, dtype=np.int32).reshape(-1, 4), "ctx": np.asarray(ctx, dtype=np.int32).reshape(-1, 3),
           "rows": np.asarray(rows, dtype=np.int32)}
    return arr, {"n_ctx": at, "max_ctx": max((c[1] for c in ctx), default=0), "rows_kv": kv}


def tiles_ok(sp: LatentHeads, dtype, ldo: int) -> bool:
    """Sizes the prompt tiles take (others run row by row)."""
    return (dtype == torch.bfloat16 and not any(n % 8 for n in (sp.dim, sp.rot_dim, sp.vdim, sp.kv_rank))
            and sp.dim + sp.rot_dim <= 256 and sp.vdim <= 256 and ldo % 4 == 0 and sp.scale > 0)


def attend_prompts(sp: LatentHeads, wt: LatentWeights, q, pages, table, pos, slots, out, ukv, b: Prompts, linear):
    """The portions of ``b.tiles`` over keys and values expanded from their contexts (which the pages hold):
    ``ukv`` [H (dim + vdim), kv_rank] = W_uk over W_uv, through ``linear(x, w)``."""
    T, H = q.shape[0], sp.heads
    assert native_dt(q, pages, wt.sink, out, ukv) == 1 and q.is_contiguous() and q.shape[1] == H * (sp.dim + sp.rot_dim)
    assert out.stride(1) == 1 and out.shape == (T, H * sp.vdim) and ukv.shape == (H * (sp.dim + sp.vdim), sp.kv_rank)
    assert b.tiles.dtype == b.ctx.dtype == torch.int32 and b.tiles.is_contiguous() and b.ctx.is_contiguous()
    a = _base(sp, wt, pages, table, pos, slots, T)
    rows = torch.empty(b.n_ctx, sp.row, device=q.device, dtype=q.dtype)
    P, LL, I = ctypes.c_void_p, ctypes.c_longlong, ctypes.c_int
    fn = _lib.require().kca_latent_gather
    fn.argtypes, fn.restype = [P, LL, P, I, I, I, P, I, I, P, P], I
    rc = fn(a.kc, a.k_sp, a.table, a.tstride, a.shift, sp.row, b.ctx.data_ptr(), b.ctx.shape[0], b.max_ctx, rows.data_ptr(),
            _lib.stream())
    if rc != 0:
        raise RuntimeError(f"kca_latent_gather returned status {rc} (unsupported shape/arguments)")
    _lib.LAUNCHES[0] += 1
    kv = linear(rows[:, :sp.kv_rank], ukv)
    assert kv.stride(1) == 1
    a.q, a.kv, a.ldkv, a.kr, a.tiles = q.data_ptr(), kv.data_ptr(), kv.stride(0), rows.data_ptr(), b.tiles.data_ptr()
    a.sink, a.out, a.ldo = wt.sink.data_ptr(), out.data_ptr(), out.stride(0)
    _call("kca_latent_tiles", a, b.tiles.shape[0])
    return out


def head_mm(x, hx: int, w, y, row_of: torch.Tensor | None = None):
    """y[b, h, :] = w[h] x[row_of[b], h, :K], x heads ``hx`` columns apart, w [H, N, K]."""
    H, N, K = w.shape
    code = native_dt(x, w, y)
    assert x.stride(1) == 1 and (H - 1) * hx + K <= x.shape[1] and y.is_contiguous() and y.shape[1] == H * N
    assert row_of is None or row_of.dtype == torch.int32
    assert y.shape[0] == (x.shape[0] if row_of is None else row_of.shape[0])
    P, LL, I = ctypes.c_void_p, ctypes.c_longlong, ctypes.c_int
    args = (x.data_ptr(), x.stride(0), hx, w.data_ptr(), y.data_ptr(), y.stride(0), N, y.shape[0], H, N, K,
            _lib.ptr(row_of), _lib.stream())
    types = [P, LL, I, P, P, LL, I, I, I, I, I, P, P]
    rc = 10
    if code == 1:
        fn = _lib.require().kca_head_mm_mfma
        fn.argtypes, fn.restype = types, I
        rc = fn(*args)
    if rc == 10:
        fn = _lib.require().kca_head_mm
        fn.argtypes, fn.restype = [I] + types, I
        rc = fn(code, *args)
    if rc != 0:
        raise RuntimeError(f"kca_head_mm returned status {rc} (unsupported shape/arguments)")
    _lib.LAUNCHES[0] += 1
    return y


def _reference(sp, wt, q, pages, table, pos, slots, out, rows):
    H, D, C = sp.heads, sp.dim, sp.kv_rank
    qf = q.float().view(-1, H, D + sp.rot_dim)
    qr = rotate(sp, wt, qf[..., D:], pos[:qf.shape[0]])
    for t in rows:
        row = gather_kv(pages, int(slots[t]), int(pos[t]) + 1, table).float()[0]      # [n, C + R]
        qa = (wt.wuk_t.float() @ qf[t, :, :D, None])[..., 0]                           # [H, C]
        s = (qa @ row[:, :C].t() + qr[t] @ row[:, C:].t()) * sp.scale
        s = torch.softmax(torch.cat([s, wt.sink.float()[:, None]], 1), -1)[:, :-1]
        out[t] = (wt.wuv.float() @ (s @ row[:, :C])[..., None])[..., 0].reshape(-1).to(out.dtype)
    return out


__all__ = ["LatentHeads", "LatentWeights", "Prompts", "latent_append", "attend_rows", "attend_prompts", "plan_prompts",
           "tiles_ok", "rows_plan", "head_mm", "rotate"]
