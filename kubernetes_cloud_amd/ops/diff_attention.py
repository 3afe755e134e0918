"""Differential attention over the paged cache (``csrc/kernels/diff_attn.hip``).

Every query head runs two softmax maps over the same values and keeps their difference, normalised per head:

    o = a_1 - lambda a_2,   o <- o / sqrt(mean(o^2) + eps) * gain

with scores q . k * scale * (1 + coef ln(floor((pos + 1) / every) + 1)). Cache layout: K pages
[pages, 2G, PS, dim] (key head 2g + i: map i of group g), V pages [pages, G, PS, vdim].
"""
from __future__ import annotations

import ctypes
import dataclasses
import math

import numpy as np
import torch

from . import _lib
from .decode import decode_chunk, gather_kv
from .rms_shift import native_dt

TILE = 128        # query rows of a matrix-core workgroup
MAX_SPLITS = 256  # key splits the rows kernel merges


class _Args(ctypes.Structure):
    _P, _LL, _I, _F = ctypes.c_void_p, ctypes.c_longlong, ctypes.c_int, ctypes.c_float
    _fields_ = [("qkv", _P), ("ld", _LL), ("kc", _P), ("vc", _P), ("k_sp", _LL), ("v_sp", _LL), ("table", _P),
                ("tstride", _I), ("shift", _I), ("pos", _P), ("slot", _P), ("out", _P), ("ldo", _LL), ("H", _I),
                ("G", _I), ("dim", _I), ("vdim", _I), ("scale", _F), ("coef", _F), ("every", ctypes.c_double),
                ("lam", _F), ("eps", _F), ("gain", _F), ("append", _I), ("nsplit", _I), ("chunk", _I), ("ws", _P),
                ("cnt", _P), ("tiles", _P), ("row_of", _P)]


@dataclasses.dataclass(frozen=True)
class DiffHeads:
    """Sizes and constants of one layer's attention."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    lam: float
    gain: float
    eps: float
    coef: float = 0.0
    every: float = 0.0   # 0: no query temperature

    @property
    def rows(self) -> int:  # width of the [q | k | v] projection
        return 2 * self.heads * self.dim + 2 * self.kv_heads * self.dim + self.kv_heads * self.vdim


def plan_tiles(entries) -> np.ndarray:
    """[(row0, rows, pos0, slot)] -> query tiles int32 [n, 4], the longest key ranges first."""
    out = [(r0 + i, min(TILE, n - i), p0 + i, s) for r0, n, p0, s in entries for i in range(0, n, TILE)]
    return np.asarray(sorted(out, key=lambda t: -(t[2] + t[1])), dtype=np.int32).reshape(-1, 4)


def tiles_ok(sp: DiffHeads, dtype, page_size: int, ldo: int) -> bool:
    """Shapes the matrix-core kernel takes (others run the rows kernel)."""
    return (dtype == torch.bfloat16 and sp.dim % 8 == 0 and sp.vdim % 8 == 0 and sp.dim <= 128 and sp.vdim <= 256
            and sp.rows % 8 == 0 and page_size >= 32 and ldo % 4 == 0)


def _abi():
    fn = _lib.require().kca_diff_attn_abi
    if fn() != ctypes.sizeof(_Args):
        raise RuntimeError(f"kca_diff_attn descriptor: C {fn()} bytes, ctypes {ctypes.sizeof(_Args)}")


def _args(sp: DiffHeads, qkv, k_pages, v_pages, table, pos, slots, out=None) -> _Args:
    PS = k_pages.shape[2]
    assert qkv.stride(1) == 1 and qkv.shape[1] == sp.rows
    assert k_pages.is_contiguous() and k_pages.shape[1:] == (2 * sp.kv_heads, PS, sp.dim)
    assert v_pages.is_contiguous() and v_pages.shape[1:] == (sp.kv_heads, PS, sp.vdim)
    assert v_pages.shape[0] == k_pages.shape[0] and PS >= 16 and PS & (PS - 1) == 0
    assert table.dtype == torch.int32 and table.is_contiguous()
    assert pos.dtype == torch.int32 and slots.dtype == torch.int32 and pos.shape[0] >= qkv.shape[0]
    _abi()
    a = _Args()
    a.qkv, a.ld = qkv.data_ptr(), qkv.stride(0)
    a.kc, a.vc, a.k_sp, a.v_sp = k_pages.data_ptr(), v_pages.data_ptr(), k_pages.stride(0), v_pages.stride(0)
    a.table, a.tstride, a.shift = table.data_ptr(), table.stride(0), PS.bit_length() - 1
    a.pos, a.slot = pos.data_ptr(), slots.data_ptr()
    if out is not None:
        assert out.stride(1) == 1 and out.shape == (qkv.shape[0], sp.heads * sp.vdim)
        a.out, a.ldo = out.data_ptr(), out.stride(0)
    a.H, a.G, a.dim, a.vdim, a.scale = sp.heads, sp.kv_heads, sp.dim, sp.vdim, sp.scale
    a.coef, a.every, a.lam, a.eps, a.gain = sp.coef, sp.every, sp.lam, sp.eps, sp.gain
    return a


def _fn(name, argtypes):
    fn = getattr(_lib.require(), name)
    fn.argtypes, fn.restype = argtypes, ctypes.c_int
    return fn


def _check(name, rc):
    if rc != 0:
        raise RuntimeError(f"{name} returned status {rc} (unsupported shape/arguments)")
    _lib.LAUNCHES[0] += 1
    if _lib.SYNC_LAUNCH:
        torch.cuda.synchronize()


def append(sp: DiffHeads, qkv, k_pages, v_pages, table, pos, slots):
    """K / V of every row of ``qkv`` into its page."""
    code = native_dt(qkv, k_pages, v_pages)
    if code is None:
        T, H, G, D = qkv.shape[0], sp.heads, sp.kv_heads, sp.dim
        k = qkv[:, 2 * H * D:2 * (H + G) * D].reshape(T, 2 * G, D)
        v = qkv[:, 2 * (H + G) * D:].reshape(T, G, sp.vdim)
        PS = k_pages.shape[2]
        pg = table.long()[slots.long()[:T], pos.long()[:T] // PS]
        k_pages[pg, :, pos.long()[:T] % PS] = k
        v_pages[pg, :, pos.long()[:T] % PS] = v
        return
    a = _args(sp, qkv, k_pages, v_pages, table, pos, slots)
    _check("kca_diff_append", _fn("kca_diff_append", [ctypes.c_void_p, ctypes.c_int, ctypes.c_int, ctypes.c_void_p])(
        ctypes.addressof(a), code, qkv.shape[0], _lib.stream()))


def rows_plan(sp: DiffHeads, rows: int, max_kv: int, dtype) -> tuple[int, int, int, int]:
    """(splits, keys per split, workspace floats, counters) of the rows kernel."""
    hg = sp.heads // sp.kv_heads
    vec = sp.dim % 8 == 0 and sp.vdim % 8 == 0 and sp.rows % 8 == 0
    rb = 4 if vec and hg > 1 else 1
    sub = -(-hg // rb)
    blocks = rows * sp.kv_heads * sub
    chunk = max(decode_chunk(rows, sp.kv_heads * sub, max_kv), -(-max_kv // MAX_SPLITS))
    n = -(-max_kv // chunk)
    return n, chunk, (blocks * n * 2 * rb * (sp.vdim + 2) if n > 1 else 0), blocks


def attend_rows(sp: DiffHeads, qkv, k_pages, v_pages, table, pos, slots, out, max_kv: int, *, fused_append: bool,
                row_of: torch.Tensor | None = None, ws: torch.Tensor | None = None, cnt: torch.Tensor | None = None):
    """One query token per row, over the row's own keys [0, pos]. ``fused_append``: the row's k / v come
    from ``qkv`` and are stored on the way (single-token entries only); else the pages hold them already.
    ``row_of``: only these rows."""
    code = native_dt(qkv, k_pages, v_pages, out)
    if code is None:
        if fused_append:
            append(sp, qkv, k_pages, v_pages, table, pos, slots)
        return _reference(sp, qkv, k_pages, v_pages, table, pos, slots, out,
                          range(qkv.shape[0]) if row_of is None else row_of.tolist())
    n = qkv.shape[0] if row_of is None else row_of.shape[0]
    splits, chunk, wsf, blocks = rows_plan(sp, n, max_kv, qkv.dtype)
    if splits > 1:
        if ws is None or ws.numel() < wsf:
            ws = torch.empty(wsf, device=qkv.device, dtype=torch.float32)
        if cnt is None or cnt.numel() < blocks:
            cnt = torch.zeros(blocks, device=qkv.device, dtype=torch.int32)
    a = _args(sp, qkv, k_pages, v_pages, table, pos, slots, out)
    a.append, a.nsplit, a.chunk, a.row_of = int(fused_append), splits, chunk, _lib.ptr(row_of)
    a.ws, a.cnt = _lib.ptr(ws), _lib.ptr(cnt)
    assert row_of is None or row_of.dtype == torch.int32
    _check("kca_diff_rows", _fn("kca_diff_rows", [ctypes.c_void_p, ctypes.c_int, ctypes.c_int, ctypes.c_longlong,
                                                  ctypes.c_longlong, ctypes.c_int, ctypes.c_void_p])(
        ctypes.addressof(a), code, n, ws.numel() if ws is not None else 0, cnt.numel() if cnt is not None else 0,
        int(max_kv), _lib.stream()))
    return out


def attend_tiles(sp: DiffHeads, qkv, k_pages, v_pages, table, pos, slots, out, tiles: torch.Tensor):
    """Prompt portions (``plan_tiles``) on the matrix cores; their K / V are in the pages (``append``)."""
    assert native_dt(qkv, k_pages, v_pages, out) == 1 and tiles.dtype == torch.int32 and tiles.is_contiguous()
    a = _args(sp, qkv, k_pages, v_pages, table, pos, slots, out)
    a.tiles = tiles.data_ptr()
    _check("kca_diff_tiles", _fn("kca_diff_tiles", [ctypes.c_void_p, ctypes.c_int, ctypes.c_void_p])(
        ctypes.addressof(a), tiles.shape[0], _lib.stream()))
    return out


def _reference(sp, qkv, k_pages, v_pages, table, pos, slots, out, rows):
    H, G, D, E = sp.heads, sp.kv_heads, sp.dim, sp.vdim
    for t in rows:
        p, s = int(pos[t]), int(slots[t])
        f = sp.scale
        if sp.every > 0:
            f *= 1 + sp.coef * math.log(math.floor((p + 1) / sp.every) + 1)
        q = qkv[t, :2 * H * D].float().view(G, H // G, 2, D) * f
        k = gather_kv(k_pages, s, p + 1, table).float().view(G, 2, p + 1, D)
        v = gather_kv(v_pages, s, p + 1, table).float()                             # [G, n, E]
        w = torch.softmax(torch.matmul(q.permute(0, 2, 1, 3), k.transpose(-1, -2)), -1)  # [G, 2, R, n]
        a = torch.matmul(w, v[:, None])                                               # [G, 2, R, E]
        o = (a[:, 0] - sp.lam * a[:, 1]).reshape(H, E)
        o = o * torch.rsqrt((o * o).mean(-1, keepdim=True) + sp.eps) * sp.gain
        out[t] = o.reshape(-1).to(out.dtype)
    return out


__all__ = ["DiffHeads", "append", "attend_rows", "attend_tiles", "plan_tiles", "rows_plan", "tiles_ok", "TILE"]
