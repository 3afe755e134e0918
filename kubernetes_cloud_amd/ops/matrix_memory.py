"""Matrix memory with exponential gates (mLSTM) over a flat batch of sequence portions
(``csrc/kernels/matrix_memory.hip``).

Per head, with log gates i = cap tanh((x_i + b_i) / cap) and f = log sigmoid(cap tanh((x_f + b_f) / cap)), a state S
[dim, vdim], a normaliser n [dim] and a running maximum m of a sequence follow

    m_t = max(f + m_(t-1), i),  w = e^(f + m_(t-1) - m_t),  p = e^(i - m_t)
    S_t = w S_(t-1) + p k v^T,  n_t = w n_(t-1) + p k
    o_t = S_t^T q / (max(|n_t . q|, e^(-m_t)) + 1e-6),      q = dim^(-1/2) (W_q h)

and the read-out is RMS-normed per head, times a gain, times sigmoid(g), times ``mul``. The projections are column blocks
of one buffer; gates, state and norms are fp32. A sequence's state lives in row ``slot`` of ``MemoryState`` and counts
as zero at position 0.
"""
from __future__ import annotations

import ctypes
import dataclasses

import torch

from . import _lib
from .delta_rule import CHUNK, Portions, _call
from .rms_shift import native_dt


_P, _LL, _I, _F = ctypes.c_void_p, ctypes.c_longlong, ctypes.c_int, ctypes.c_float


class _Args(ctypes.Structure):
    _fields_ = [("x", _P), ("ld", _LL), *[(n, _I) for n in ("o_q", "o_k", "o_v", "o_g", "o_i", "o_f", "H", "dk", "dv")],
                ("ib", _P), ("fb", _P), ("gain", _P), ("cap", _F), ("qscale", _F), ("eps", _F), ("mul", _F),
                *[(n, _P) for n in ("state", "norm", "top", "norm1", "top1", "pos", "slot", "e1", "out")], ("ldo", _LL),
                *[(n, _P) for n in ("o", "ent", "ck", "en", "am", "kt", "gd")]]


@dataclasses.dataclass(frozen=True)
class MemoryHeads:
    """Sizes and constants of one layer. ``at``: first columns of q, k, v, g and of the input and forget gates."""
    heads: int
    dim: int
    vdim: int
    at: tuple
    gate_cap: float
    eps: float
    mul: float = 1.0


@dataclasses.dataclass(frozen=True)
class MemoryWeights:
    """Gate biases [H] and the gain of the heads' norm [H vdim]."""
    i_bias: torch.Tensor
    f_bias: torch.Tensor
    gain: torch.Tensor


@dataclasses.dataclass(frozen=True)
class MemoryState:
    """fp32, one row a slot: S [H dim vdim], n [H dim], m [H]."""
    s: torch.Tensor
    n: torch.Tensor
    m: torch.Tensor


def chunks_ok(sp: MemoryHeads, dtype) -> bool:
    """Sizes the chunked matrix-core kernels take (others, and fp32, run token by token)."""
    return dtype == torch.bfloat16 and sp.dim % 8 == 0 and sp.vdim % 8 == 0 and sp.dim <= 128


def _args(sp: MemoryHeads, wt: MemoryWeights, x, st: MemoryState, pos, slots, out) -> tuple[_Args, int]:
    H, D, E = sp.heads, sp.dim, sp.vdim
    code = native_dt(x, wt.i_bias, wt.f_bias, wt.gain, out)
    assert x.stride(1) == 1 and out.stride(1) == 1 and out.shape == (x.shape[0], H * E)
    assert all(0 <= o and o + n <= x.shape[1] for o, n in zip(sp.at, (H * D, H * D, H * E, H * E, H, H)))
    assert all(t.is_contiguous() and t.dtype == torch.float32 and t.shape[1] == w
               for t, w in ((st.s, H * D * E), (st.n, H * D), (st.m, H)))
    assert all(t.is_contiguous() and t.numel() == n for t, n in ((wt.i_bias, H), (wt.f_bias, H), (wt.gain, H * E)))
    assert all(t.dtype == torch.int32 and t.shape[0] >= x.shape[0] for t in (pos, slots))
    a = _Args()
    if code is None:
        return a, None
    if _lib.require().kca_memory_abi() != ctypes.sizeof(_Args):
        raise RuntimeError("kca_memory descriptor: C and ctypes sizes differ")
    a.x, a.ld = x.data_ptr(), x.stride(0)
    a.o_q, a.o_k, a.o_v, a.o_g, a.o_i, a.o_f = sp.at
    a.H, a.dk, a.dv = H, D, E
    a.ib, a.fb, a.gain = wt.i_bias.data_ptr(), wt.f_bias.data_ptr(), wt.gain.data_ptr()
    a.cap, a.qscale, a.eps, a.mul = sp.gate_cap, D ** -0.5, sp.eps, sp.mul
    a.state, a.norm, a.top = st.s.data_ptr(), st.n.data_ptr(), st.m.data_ptr()
    a.pos, a.slot, a.out, a.ldo = pos.data_ptr(), slots.data_ptr(), out.data_ptr(), out.stride(0)
    return a, code


def memory_step(sp: MemoryHeads, wt: MemoryWeights, x, st: MemoryState, pos, slots, out) -> torch.Tensor:
    """One token per row: row b continues ``slots[b]`` at ``pos[b]``."""
    a, code = _args(sp, wt, x, st, pos, slots, out)
    if code is None:
        return _reference(sp, wt, x, st, [(i, 1, int(pos[i]), int(slots[i])) for i in range(x.shape[0])], out)
    _call("kca_memory_step", a, code, x.shape[0])
    return out


def memory_portions(sp: MemoryHeads, wt: MemoryWeights, x, st: MemoryState, b: Portions, out) -> torch.Tensor:
    """Portions of any sizes."""
    a, code = _args(sp, wt, x, st, b.pos, b.slots, out)
    if code is None:
        return _reference(sp, wt, x, st, b.ent[:, :4].tolist(), out)
    T, H, dev = x.shape[0], sp.heads, x.device
    assert all(t.dtype == torch.int32 and t.is_contiguous() for t in (b.e1, b.ent, b.short, b.chunked, b.chunks))
    o = torch.empty(T, H * sp.vdim, device=dev, dtype=x.dtype)
    n1, m1 = torch.empty_like(st.n), torch.empty_like(st.m)
    a.o, a.e1, a.norm1, a.top1 = o.data_ptr(), b.e1.data_ptr(), n1.data_ptr(), m1.data_ptr()
    chunked = chunks_ok(sp, x.dtype) and b.chunks.shape[0] > 0
    if chunked:
        nc, DK = b.chunks.shape[0], (64 if sp.dim <= 64 else 128)
        am, kt = (torch.empty(nc * H * n * CHUNK, device=dev, dtype=torch.bfloat16) for n in (CHUNK, DK))
        gd = torch.empty(nc * H * (3 * CHUNK + DK), device=dev, dtype=torch.float32)
        a.ck, a.en, a.am, a.kt, a.gd = (t.data_ptr() for t in (b.chunks, b.chunked, am, kt, gd))
        _call("kca_memory_chunks", a, nc, b.chunked.shape[0])
    ent = b.short if chunked else b.ent
    if ent.shape[0]:
        a.ent = ent.data_ptr()
        _call("kca_memory_scan", a, code, ent.shape[0])
    _call("kca_memory_gate", a, code, T)
    return out


def _reference(sp, wt, x, st, entries, out):
    H, D, E = sp.heads, sp.dim, sp.vdim
    T, xf = x.shape[0], x.float()
    col = lambda j, n: xf[:, sp.at[j]:sp.at[j] + n]  # noqa: E731
    cap = lambda z, b: sp.gate_cap * torch.tanh((z + b.float()) / sp.gate_cap)  # noqa: E731
    q, k, v = col(0, H * D).reshape(T, H, D) * D ** -0.5, col(1, H * D).reshape(T, H, D), col(2, H * E).reshape(T, H, E)
    gi, gf = cap(col(4, H), wt.i_bias), torch.nn.functional.logsigmoid(cap(col(5, H), wt.f_bias))
    o = torch.empty(T, H, E)
    for r0, count, pos, slot in entries:
        S, n, m = (t[slot].clone() if pos > 0 else torch.zeros_like(t[slot]) for t in (st.s, st.n, st.m))
        S, n = S.view(H, D, E), n.view(H, D)
        for t in range(r0, r0 + count):
            top = torch.maximum(gf[t] + m, gi[t])
            w, p, m = torch.exp(gf[t] + m - top), torch.exp(gi[t] - top), top
            S = w[:, None, None] * S + (p[:, None] * k[t])[..., None] * v[t][:, None]
            n = w[:, None] * n + p[:, None] * k[t]
            o[t] = (S * q[t][..., None]).sum(1) / (torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6)[:, None]
        st.s[slot], st.n[slot], st.m[slot] = S.reshape(-1), n.reshape(-1), m
    y = (o * torch.rsqrt((o * o).mean(-1, keepdim=True) + sp.eps)).reshape(T, H * E) * wt.gain.float()
    out.copy_(y * torch.sigmoid(col(3, H * E)) * sp.mul)
    return out


__all__ = ["MemoryHeads", "MemoryWeights", "MemoryState", "chunks_ok", "memory_step", "memory_portions"]
