"""Residual add + RMS norm + token shift over a flat batch of sequence portions (``csrc/kernels/rms_shift.hip``).

    x_t  = x_in_t + m * (a_t + sum_k y[inv[t, k]])          fp32 residual stream
    h_t  = x_t / sqrt(mean(x_t^2) + eps) * g
    hs_t = h_t + (h_(t-1) - h_t) * mu

bf16 and fp32 GPU tensors run the kernel; CPU tensors run the reference below.
"""
from __future__ import annotations

import dataclasses

import torch

from . import _lib

DT = {torch.float32: 0, torch.bfloat16: 1}


def native_dt(*tensors) -> int | None:
    """Kernel type code of GPU tensors (fp32 / bf16, all alike), None for CPU tensors."""
    ts = [t for t in tensors if t is not None]
    if not ts[0].is_cuda:
        return None
    dt = ts[0].dtype
    if dt not in DT or any(t.dtype != dt or not t.is_cuda for t in ts):
        raise TypeError(f"these kernels take fp32 or bf16 tensors of one type, got {[t.dtype for t in ts]}")
    return DT[dt]


@dataclasses.dataclass
class Branch:
    """What a layer adds to the residual stream: ``a`` [T, d], plus (routed experts) the sorted expert rows
    ``y`` [n, d] summed through ``inv`` [T, top]."""
    a: torch.Tensor
    y: torch.Tensor | None = None
    inv: torch.Tensor | None = None


def rows_per_block(T: int) -> int:
    """Rows a workgroup walks: a longer walk recomputes fewer left neighbours, a short batch needs the spread."""
    return 8 if T >= 4096 else 4 if T >= 1024 else 2 if T >= 512 else 1


def rms_shift(x: torch.Tensor | None, branch: Branch | None, m: float, gain: torch.Tensor, eps: float, *,
              embed: torch.Tensor | None = None, tokens: torch.Tensor | None = None,
              shift: torch.Tensor | None = None, prev: torch.Tensor | None = None,
              prev_idx: torch.Tensor | None = None, pos: torch.Tensor | None = None,
              flags: torch.Tensor | None = None, state: torch.Tensor | None = None,
              slots: torch.Tensor | None = None, rows: torch.Tensor | None = None, keep_x: bool = True):
    """-> (x_out fp32 | None, h, hs | None). ``x`` None: the stream starts at ``embed[tokens]``.

    ``prev`` [*, d] fp32 holds the carried rows, ``prev_idx`` [T] the row of an entry-first token; ``flags``
    [T] int32 bit 0 / 1: the entry's first / last token (None: every row is both). ``state`` [slots, d]
    receives each entry's last h. ``rows``: only these tokens (no shift, no x_out)."""
    d = gain.shape[0] if (x is None and embed is None) else (embed if x is None else x).shape[1]
    T = rows.shape[0] if rows is not None else (tokens if x is None else x).shape[0]
    dt_ref = embed if embed is not None else gain
    keep_x = keep_x and rows is None
    a = branch.a if branch is not None else None
    y = branch.y if branch is not None else None
    inv = branch.inv if branch is not None else None
    code = native_dt(gain, embed, a, y, shift)
    dev, dtype = gain.device, dt_ref.dtype
    if code is None:
        return _reference(x, a, y, inv, m, gain, eps, embed, tokens, shift, prev, prev_idx, pos, flags, state, slots,
                          rows, keep_x, dtype)
    assert a is None or (a.stride(1) == 1 and a.shape[1] == d)
    assert y is None or (y.is_contiguous() and y.shape[1] == d and inv.is_contiguous() and inv.dtype == torch.int32)
    assert x is None or (x.is_contiguous() and x.dtype == torch.float32)
    assert embed is None or embed.is_contiguous()
    assert tokens is None or tokens.dtype == torch.int64
    if shift is not None:
        assert prev.is_contiguous() and prev.dtype == torch.float32 and prev.shape[1] == d
        assert state.is_contiguous() and state.dtype == torch.float32 and state.shape[1] == d
        assert all(t.dtype == torch.int32 and t.shape[0] >= T for t in (prev_idx, pos, slots))
    x_out = torch.empty(T, d, device=dev, dtype=torch.float32) if keep_x else None
    h = torch.empty(T, d, device=dev, dtype=dtype)
    hs = torch.empty(T, d, device=dev, dtype=dtype) if shift is not None else None
    p = _lib.ptr
    _lib.call("kca_rms_shift", code, p(x), p(embed if x is None else None), p(tokens), p(a),
              a.stride(0) if a is not None else 0, p(y), p(inv), inv.shape[1] if inv is not None else 0, float(m),
              p(gain), int(gain.numel() > 1), float(eps), p(shift), p(prev), p(prev_idx), p(pos), p(flags), p(state),
              p(slots), p(rows), p(x_out), p(h), p(hs), T, d, rows_per_block(T), _lib.stream())
    return x_out, h, hs


def _reference(x, a, y, inv, m, gain, eps, embed, tokens, shift, prev, prev_idx, pos, flags, state, slots, rows,
               keep_x, dtype):
    x = embed[tokens].float() if x is None else x
    add = 0.0
    if a is not None:
        add = a.float()
    if y is not None:
        add = add + y.float()[inv.long()].sum(1)
    x = x + m * add
    if rows is not None:
        x = x[rows.long()]
    h = x * torch.rsqrt((x * x).mean(-1, keepdim=True) + eps) * gain.float().reshape(-1)
    hs = None
    if shift is not None:
        T = x.shape[0]
        fl = torch.full((T,), 3, dtype=torch.int32) if flags is None else flags
        first = (fl & 1).bool()
        carried = prev[prev_idx.long()] * (pos > 0)[:, None]
        left = torch.cat([torch.zeros_like(h[:1]), h[:-1]])
        left = torch.where(first[:, None], carried, left)
        hs = (h + (left - h) * shift.float()).to(dtype)
        last = (fl & 2).bool()
        state[slots.long()[last]] = h[last]
    return (x if keep_x else None), h.to(dtype), hs


__all__ = ["Branch", "rms_shift", "native_dt", "DT"]
