"""Gated linear recurrence (minGRU form) over a flat batch of sequence portions (``csrc/kernels/gated_scan.hip``).

    z = sigmoid(zx + bz),  u = ux + bx,  c = u + 1/2 (u >= 0) | sigmoid(u) (u < 0)
    S_t = (1 - z) S_(t-1) + z c,    y_t = S_t * silu(g_t)

``zxg`` rows hold the three projections side by side. The fp32 state of a sequence lives in row ``slot`` of
``state`` and counts as zero at position 0.
"""
from __future__ import annotations

import numpy as np
import torch

from . import _lib
from .rms_shift import native_dt

MIN_CHUNK = 32
MAX_CHUNKS = 64  # per portion: a chunk folds its predecessors' maps one by one


def plan_chunks(entries) -> tuple[np.ndarray, bool]:
    """[(row0, rows, pos0, slot)] -> chunk descriptors int32 [n, 6] and whether a portion has several chunks."""
    longest = max(n for _, n, _, _ in entries)
    size = MIN_CHUNK
    while size * MAX_CHUNKS < longest:
        size *= 2
    out = []
    for row0, n, pos0, slot in entries:
        nc = -(-n // size)
        out += [(row0 + i * size, min(size, n - i * size), i, nc, pos0 + i * size, slot) for i in range(nc)]
    return np.asarray(out, dtype=np.int32), any(c[3] > 1 for c in out)


def gated_scan(zxg: torch.Tensor, bz: torch.Tensor, bx: torch.Tensor, state: torch.Tensor, out: torch.Tensor,
               chunks: torch.Tensor, multi: bool, ws: torch.Tensor | None = None) -> torch.Tensor:
    """Portions cut in ``chunks`` (``plan_chunks``, on the device)."""
    W = bz.shape[0]
    code = native_dt(zxg, bz, bx, out)
    assert zxg.stride(1) == 1 and zxg.shape[1] == 3 * W and out.stride(1) == 1 and state.shape[1] == W
    if code is None:
        return _reference(zxg, bz, bx, state, out, _entries(chunks))
    assert chunks.dtype == torch.int32 and chunks.is_contiguous() and state.dtype == torch.float32
    n = chunks.shape[0]
    need = n * 3 * W if multi else 0
    if need and (ws is None or ws.numel() < need):
        ws = torch.empty(need, device=zxg.device, dtype=torch.float32)
    _lib.call("kca_gated_scan", code, zxg.data_ptr(), zxg.stride(0), bz.data_ptr(), bx.data_ptr(), out.data_ptr(),
              out.stride(0), state.data_ptr(), _lib.ptr(ws), ws.numel() if ws is not None else 0, chunks.data_ptr(), n,
              int(multi), W, _lib.stream())
    return out


def gated_step(zxg: torch.Tensor, bz: torch.Tensor, bx: torch.Tensor, state: torch.Tensor, out: torch.Tensor,
               pos: torch.Tensor, slots: torch.Tensor) -> torch.Tensor:
    """One token per row: row b continues ``slots[b]`` at ``pos[b]``."""
    W = bz.shape[0]
    code = native_dt(zxg, bz, bx, out)
    assert zxg.stride(1) == 1 and zxg.shape[1] == 3 * W and out.stride(1) == 1 and state.shape[1] == W
    if code is None:
        return _reference(zxg, bz, bx, state, out,
                          [(i, 1, int(p), int(s)) for i, (p, s) in enumerate(zip(pos, slots))])
    assert pos.dtype == torch.int32 and slots.dtype == torch.int32
    _lib.call("kca_gated_step", code, zxg.data_ptr(), zxg.stride(0), bz.data_ptr(), bx.data_ptr(), out.data_ptr(),
              out.stride(0), state.data_ptr(), pos.data_ptr(), slots.data_ptr(), zxg.shape[0], W, _lib.stream())
    return out


def _entries(chunks):
    return [(r, n, p, s) for r, n, _, _, p, s in chunks.tolist()]  # in order: a chunk continues its slot


def _reference(zxg, bz, bx, state, out, entries):
    W = bz.shape[0]
    z = torch.sigmoid(zxg[:, :W].float() + bz.float())
    u = zxg[:, W:2 * W].float() + bx.float()
    zc = z * torch.where(u >= 0, u + 0.5, torch.sigmoid(u))
    g = zxg[:, 2 * W:].float()
    g = g * torch.sigmoid(g)
    for row0, n, pos, slot in entries:
        S = state[slot].clone() if pos > 0 else torch.zeros(W)
        for t in range(row0, row0 + n):
            S = (1 - z[t]) * S + zc[t]
            out[t] = (S * g[t]).to(out.dtype)
        state[slot] = S
    return out


__all__ = ["gated_scan", "gated_step", "plan_chunks"]
