"""Norms before and after a sublayer around an fp32 residual stream (``csrc/kernels/norm_residual.hip``).

    x_t = x_in_t + ls * N(a_t + b; gb)        what a sublayer adds, normed and scaled
    h_t = N(x_t; g)                           what the next sublayer reads

N: layer norm without a bias, or RMS norm. Pre-norm layers (``prenorm``, RMS throughout) add a sublayer's output
as it is, or the weighted sum of two normed ones, and norm with a gain stored around zero:

    x_t = src_t + a_t   |   src_t + mul * (N(a_t; ga) + N(b_t; gb)),      h_t = N(x_t; 1 + g)

Post-norm layers (``postnorm``, RMS, gains of one number) norm what a sublayer adds -- the sum of its rows, of routed
experts' rows and of the stream itself where an identity expert was chosen -- and hand the stream on as it is:

    x_t = src_t + ga N(a_t + sum_k y[inv[t, k]] + (sum of the weights of identity experts) src_t),      h_t = x_t

bf16 and fp32 GPU tensors run the kernels; CPU tensors run the references below.
"""
from __future__ import annotations

import ctypes
import dataclasses

import torch

from . import _lib
from .rms_shift import DT, native_dt


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


@dataclasses.dataclass
class Embedded:
    """A stream that starts at ``table[tokens] * scale``."""
    table: torch.Tensor
    tokens: torch.Tensor
    scale: float = 1.0


@dataclasses.dataclass
class Rows:
    """A stream that starts at a product's rows ``a`` [T, d] plus one vector."""
    a: torch.Tensor
    vec: torch.Tensor | None = None


@dataclasses.dataclass
class NormedPair:
    """``mul * (N(a; gain_a) + N(b; gain_b))`` of two sublayers' outputs."""
    a: torch.Tensor
    gain_a: torch.Tensor
    b: torch.Tensor
    gain_b: torch.Tensor
    mul: float = 0.5


class _PreArgs(ctypes.Structure):
    _P, _LL, _F, _I = ctypes.c_void_p, ctypes.c_longlong, ctypes.c_float, ctypes.c_int
    _fields_ = [("x_in", _P), ("embed", _P), ("tokens", _P), ("escale", _F), ("base", _P), ("ldbase", _LL), ("vec", _P),
                ("a", _P), ("lda", _LL), ("ga", _P), ("b", _P), ("ldb", _LL), ("gb", _P), ("mul", _F), ("g", _P),
                ("eps", _F), ("rows", _P), ("x_out", _P), ("raw", _P), ("ldr", _LL), ("h", _P), ("T", _I), ("d", _I)]


def prenorm(src: torch.Tensor | Embedded | Rows, branch: torch.Tensor | NormedPair | None, gain: torch.Tensor | None,
            eps: float, *, raw: torch.Tensor | None = None, rows: torch.Tensor | None = None, keep_x: bool = True):
    """-> (x_out fp32 | None, h | None). ``src``: the fp32 stream, or where it starts. ``branch``: what a sublayer
    adds. ``gain``: the next norm's, minus one (None: no h). ``raw`` [T, d] (row stride free) receives x rounded to
    its type. ``rows``: only these tokens."""
    emb, prod = isinstance(src, Embedded), isinstance(src, Rows)
    data = src.table if emb else src.a if prod else src
    d = data.shape[1]
    T = rows.shape[0] if rows is not None else (src.tokens if emb else data).shape[0]
    pair = branch if isinstance(branch, NormedPair) else None
    a = pair.a if pair else branch
    ref = next(t for t in (gain, a, raw, data) if t is not None)
    code = native_dt(ref, gain, a, raw, *((data,) if emb or prod else ()), src.vec if prod else None,
                     *((pair.gain_a, pair.b, pair.gain_b) if pair else ()))
    if code is None:
        x = src.table[src.tokens].float() * src.scale if emb else src.a.float() if prod else src
        if prod and src.vec is not None:
            x = x + src.vec.float()
        if pair:
            x = x + pair.mul * (_norm(pair.a.float(), pair.gain_a, eps, False) + _norm(pair.b.float(), pair.gain_b, eps, False))
        elif a is not None:
            x = x + a.float()
        if rows is not None:
            x = x[rows.long()]
        if raw is not None:
            raw.copy_(x)
        return (x if keep_x else None), (None if gain is None else _norm(x, 1 + gain.float(), eps, False).to(ref.dtype))
    n_src = src.tokens.shape[0] if emb else data.shape[0]
    assert data.stride(1) == 1 and (prod or data.is_contiguous()) and (emb or prod or data.dtype == torch.float32)
    assert not emb or src.tokens.dtype == torch.int64
    assert all(t is None or (t.stride(1) == 1 and t.shape == (n_src, d)) for t in (a, pair.b if pair else None))
    vecs = (gain, src.vec if prod else None, *((pair.gain_a, pair.gain_b) if pair else ()))
    assert all(t is None or (t.stride(-1) == 1 and t.numel() == d) for t in vecs)
    assert raw is None or (raw.stride(1) == 1 and raw.shape == (T, d))
    assert rows is None or rows.dtype == torch.int32
    if _lib.require().kca_prenorm_abi() != ctypes.sizeof(_PreArgs):
        raise RuntimeError("kca_prenorm descriptor: C and ctypes sizes differ")
    x_out = torch.empty(T, d, device=ref.device, dtype=torch.float32) if keep_x else None
    h = torch.empty(T, d, device=ref.device, dtype=ref.dtype) if gain is not None else None
    p, k = _lib.ptr, _PreArgs()
    if emb:
        k.embed, k.tokens, k.escale = data.data_ptr(), src.tokens.data_ptr(), src.scale
    elif prod:
        k.base, k.ldbase, k.vec = data.data_ptr(), data.stride(0), p(src.vec)
    else:
        k.x_in = data.data_ptr()
    if a is not None:
        k.a, k.lda = a.data_ptr(), a.stride(0)
    if pair:
        k.ga, k.b, k.ldb, k.gb, k.mul = p(pair.gain_a), p(pair.b), pair.b.stride(0), p(pair.gain_b), pair.mul
    k.g, k.eps, k.rows, k.x_out, k.raw, k.h, k.T, k.d = p(gain), eps, p(rows), p(x_out), p(raw), p(h), T, d
    k.ldr = raw.stride(0) if raw is not None else 0
    fn = _lib.require().kca_prenorm
    fn.argtypes, fn.restype = [ctypes.c_void_p, ctypes.c_int, ctypes.c_void_p], ctypes.c_int
    _lib.call("kca_prenorm", ctypes.addressof(k), code, _lib.stream())
    return x_out, h


@dataclasses.dataclass
class NormedSum:
    """What a sublayer adds before its norm: ``a`` [T, d] and / or routed rows ``y`` [n, d] through ``inv`` [T, top]
    (-1: the stream itself, times its weight in ``wts``)."""
    gain: torch.Tensor
    a: torch.Tensor | None = None
    y: torch.Tensor | None = None
    inv: torch.Tensor | None = None
    wts: torch.Tensor | None = None


class _PostArgs(ctypes.Structure):
    _P, _LL, _F, _I = ctypes.c_void_p, ctypes.c_longlong, ctypes.c_float, ctypes.c_int
    _fields_ = [("x_in", _P), ("embed", _P), ("tokens", _P), ("escale", _F), ("a", _P), ("lda", _LL), ("y", _P), ("inv", _P),
                ("wts", _P), ("top", _I), ("ga", _P), ("g", _P), ("hmul", _F), ("eps", _F), ("rows", _P), ("x_out", _P),
                ("h", _P), ("T", _I), ("d", _I)]


def postnorm(src: torch.Tensor | Embedded, branch: NormedSum | None, eps: float, dtype, *, gain: torch.Tensor | None = None,
             mul: float = 1.0, rows: torch.Tensor | None = None, keep_x: bool = True):
    """-> (x_out fp32 | None, h of ``dtype``). ``src``: the fp32 stream, or where it starts. h: the stream rounded, or with
    ``gain`` (one number) its RMS norm times ``mul``. ``rows``: only these tokens."""
    emb = isinstance(src, Embedded)
    data = src.table if emb else src
    n_src, d = (src.tokens if emb else data).shape[0], data.shape[1]
    T = rows.shape[0] if rows is not None else n_src
    br = branch or NormedSum(None)
    assert all(t is None or t.dtype == dtype for t in (br.gain, gain, br.a, br.y, data if emb else None))
    if not data.is_cuda:
        x = src.table[src.tokens].float() * src.scale if emb else src
        if branch is not None:
            u = torch.zeros_like(x) if br.a is None else br.a.float()
            if br.y is not None:
                inv = br.inv.long()
                u = u + br.y[inv.clamp(min=0)].float().masked_fill((inv < 0)[..., None], 0.0).sum(1)
                u = u + (br.wts * (inv < 0)).sum(1, keepdim=True) * x
            x = x + _norm(u, br.gain, eps, False)
        if rows is not None:
            x = x[rows.long()]
        return (x if keep_x else None), (x if gain is None else _norm(x, gain, eps, False) * mul).to(dtype)
    assert data.is_contiguous() and (data.dtype == torch.float32 or emb) and (not emb or src.tokens.dtype == torch.int64)
    assert all(t is None or t.numel() == 1 for t in (br.gain, gain))
    assert br.a is None or (br.a.stride(1) == 1 and br.a.shape == (n_src, d))
    assert br.y is None or (br.y.is_contiguous() and br.y.shape[1] == d and br.inv.is_contiguous() and br.wts.is_contiguous()
                            and br.inv.shape == br.wts.shape and br.inv.shape[0] == n_src and br.inv.dtype == torch.int32
                            and br.wts.dtype == torch.float32)
    assert rows is None or rows.dtype == torch.int32
    if _lib.require().kca_postnorm_abi() != ctypes.sizeof(_PostArgs):
        raise RuntimeError("kca_postnorm descriptor: C and ctypes sizes differ")
    same = dtype == torch.float32 and gain is None  # the stream is already what the next product reads
    x_out = torch.empty(T, d, device=data.device, dtype=torch.float32) if keep_x or same else None
    h = None if same else torch.empty(T, d, device=data.device, dtype=dtype)
    p, k = _lib.ptr, _PostArgs()
    if emb:
        k.embed, k.tokens, k.escale = data.data_ptr(), src.tokens.data_ptr(), src.scale
    else:
        k.x_in = data.data_ptr()
    if br.a is not None:
        k.a, k.lda = br.a.data_ptr(), br.a.stride(0)
    if br.y is not None:
        k.y, k.inv, k.wts, k.top = br.y.data_ptr(), br.inv.data_ptr(), br.wts.data_ptr(), br.inv.shape[1]
    k.ga, k.g, k.hmul, k.eps, k.rows, k.x_out, k.h, k.T, k.d = (p(br.gain), p(gain), mul, eps, p(rows), p(x_out), p(h), T, d)
    fn = _lib.require().kca_postnorm
    fn.argtypes, fn.restype = [ctypes.c_void_p, ctypes.c_int, ctypes.c_void_p], ctypes.c_int
    _lib.call("kca_postnorm", ctypes.addressof(k), DT[dtype], _lib.stream())
    return x_out, (x_out if same else h)


def _norm(x, gain, eps, layer):
    if layer:
        x = x - x.mean(-1, keepdim=True)
    return x * torch.rsqrt((x * x).mean(-1, keepdim=True) + eps) * gain.float()


__all__ = ["Embedded", "NormedBranch", "NormedPair", "NormedSum", "Rows", "norm_residual", "postnorm", "prenorm"]
