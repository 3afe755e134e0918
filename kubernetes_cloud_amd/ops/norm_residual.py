"""Norms before and after a sublayer around an fp32 residual stream (``csrc/kernels/norm_residual.hip``).

    x_t = x_in_t + ls * N(a_t + b; gb)        what a sublayer adds, normed and scaled
    h_t = N(x_t; g)                           what the next sublayer reads

N: layer norm without a bias, or RMS norm. bf16 and fp32 GPU tensors run the kernel; CPU tensors run the
reference below.
"""
from __future__ import annotations

import dataclasses

import torch

from . import _lib
from .rms_shift import native_dt


@dataclasses.dataclass
class NormedBranch:
    """A sublayer's output ``a`` [T, d] (+ ``bias``), the gain of its output norm and its layer scale."""
    a: torch.Tensor
    gain: torch.Tensor
    scale: torch.Tensor | None = None
    bias: torch.Tensor | None = None


def norm_residual(x: torch.Tensor | None, branch: NormedBranch | None, gain: torch.Tensor | None, eps: float, *,
                  layer: bool = True, embed: torch.Tensor | None = None, tokens: torch.Tensor | None = None,
                  rows: torch.Tensor | None = None, keep_x: bool = True):
    """-> (x_out fp32 | None, h | None). ``x`` None: the stream starts at ``embed[tokens]``. ``rows``: only
    these tokens. ``gain`` None: no h."""
    d = (embed if x is None else x).shape[1]
    T = rows.shape[0] if rows is not None else (tokens if x is None else x).shape[0]
    ref = gain if gain is not None else branch.gain
    br = branch or NormedBranch(None, None)
    code = native_dt(ref, embed if x is None else None, gain, br.a, br.gain, br.scale, br.bias)
    if code is None:
        x = embed[tokens].float() if x is None else x
        if branch is not None:
            y = br.a.float() if br.bias is None else br.a.float() + br.bias.float()
            y = _norm(y, br.gain, eps, layer)
            x = x + (y if br.scale is None else y * br.scale.float())
        if rows is not None:
            x = x[rows.long()]
        return (x if keep_x else None), (None if gain is None else _norm(x, gain, eps, layer).to(ref.dtype))
    assert br.a is None or (br.a.stride(1) == 1 and br.a.shape[1] == d and br.gain.is_contiguous() and br.gain.numel() == d)
    assert all(t is None or (t.is_contiguous() and t.numel() == d) for t in (gain, br.scale, br.bias))
    assert x is None or (x.is_contiguous() and x.dtype == torch.float32)
    assert x is not None or (embed.is_contiguous() and tokens.dtype == torch.int64)
    assert rows is None or rows.dtype == torch.int32
    x_out = torch.empty(T, d, device=ref.device, dtype=torch.float32) if keep_x else None
    h = torch.empty(T, d, device=ref.device, dtype=ref.dtype) if gain is not None else None
    p = _lib.ptr
    _lib.call("kca_norm_residual", code, p(x), p(embed if x is None else None), p(tokens if x is None else None), p(br.a),
              br.a.stride(0) if br.a is not None else 0, p(br.bias), p(br.gain), p(br.scale), p(gain), float(eps), p(rows),
              p(x_out), p(h), T, d, int(layer), _lib.stream())
    return x_out, h


def _norm(x, gain, eps, layer):
    if layer:
        x = x - x.mean(-1, keepdim=True)
    return x * torch.rsqrt((x * x).mean(-1, keepdim=True) + eps) * gain.float()


__all__ = ["NormedBranch", "norm_residual"]
