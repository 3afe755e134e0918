"""Delta-rule token mixers over a flat batch of sequence portions (``csrc/kernels/delta_rule.h``).

Per head a state S [dk, dv] of a sequence follows

    S_t = diag(w_t) S_(t-1) + p_t (z_t^T S_(t-1)) + k_t v_t^T,     o_t = S_t^T q_t

and the read-out is RMS-normed per head, times a gain, times a sigmoid gate. Two forms make the vectors from
the projections ``x`` (column blocks named by ``DeltaHeads.at``):

* general: w = exp(-e^(-1/2) sigmoid(lw + w0)), z = u = k / sqrt(|k|^2 + 1e-6), p = -(a u), a = sigmoid(.. + b)
* channel: q, k, v through short causal convolutions and silu; unit q (times dk^(-1/2)) and k, shared by groups
  of heads; w = exp(-exp(A) softplus(lw + dt)), z = w k, p = -beta k, k <- beta k

lw is the second step of a two-step projection (general: tanh between). Vectors, state and gates are fp32.
The state of a sequence lives in row ``slot`` of ``state``; the convolution inputs of its last positions in
``ring`` (position p in row p % taps). Both count as zero at and before position 0.
"""
from __future__ import annotations

import ctypes
import dataclasses
import math

import torch

from . import _lib
from .rms_shift import native_dt


_P, _LL, _I, _F = ctypes.c_void_p, ctypes.c_longlong, ctypes.c_int, ctypes.c_float


class _Args(ctypes.Structure):
    _fields_ = [("x", _P), ("ld", _LL), *[(n, _I) for n in ("o_q", "o_k", "o_v", "o_a", "o_g", "o_w")],
                *[(n, _I) for n in ("H", "G", "dk", "dv", "taps", "rank_w", "rank_g")], ("lo_w", _P), ("lo_g", _P),
                ("dw", _P), ("ldw", _LL), ("dg", _P), ("ldg", _LL), ("w0", _P), ("ab", _P), ("conv", _P), ("gain", _P),
                ("eps", _F), ("qscale", _F), ("state", _P), ("ring", _P), ("pos", _P), ("slot", _P), ("e0", _P),
                ("e1", _P), ("out", _P), ("ldo", _LL), ("pk", _P), ("o", _P), ("ent", _P)]


@dataclasses.dataclass(frozen=True)
class DeltaHeads:
    """Sizes and constants of one layer. ``at``: first column of q, k, v, a (removal or beta), g (gate or its
    first step) and w (the decay's first step) in the projection rows."""
    general: bool
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    at: tuple
    rank_w: int
    eps: float
    taps: int = 0
    rank_g: int = 0

    @property
    def conv_channels(self) -> int:
        return 0 if self.general else 2 * self.kv_heads * self.dim + self.heads * self.vdim

    @property
    def state_width(self) -> int:
        return self.heads * self.dim * self.vdim


@dataclasses.dataclass(frozen=True)
class DeltaWeights:
    """``ab``: bias of a (general) or A per head (channel); ``lo_g``, ``conv``: channel only."""
    lo_w: torch.Tensor
    w0: torch.Tensor
    ab: torch.Tensor
    gain: torch.Tensor
    lo_g: torch.Tensor | None = None
    conv: torch.Tensor | None = None


@dataclasses.dataclass
class Portions:
    """Device arrays of a batch of portions: per row its position, slot, and the first and one-past-last row of
    its entry; ``ent`` [n, 4]: first row, rows, position of the first row, slot."""
    pos: torch.Tensor
    slots: torch.Tensor
    e0: torch.Tensor
    e1: torch.Tensor
    ent: torch.Tensor


def _args(sp: DeltaHeads, wt: DeltaWeights, x, state, ring, pos, slots, out) -> tuple[_Args, int]:
    code = native_dt(x, wt.lo_w, wt.w0, wt.ab, wt.gain, wt.lo_g, wt.conv, out)
    assert x.stride(1) == 1 and out.stride(1) == 1 and out.shape == (x.shape[0], sp.heads * sp.vdim)
    assert state.is_contiguous() and state.dtype == torch.float32 and state.shape[1] == sp.state_width
    assert all(t is None or t.is_contiguous() for t in (wt.lo_w, wt.w0, wt.ab, wt.gain, wt.lo_g, wt.conv))
    assert wt.lo_w.shape == (sp.heads * sp.dim, sp.rank_w) and wt.w0.numel() == sp.heads * sp.dim
    ends = (sp.kv_heads * sp.dim,) * 2 + (sp.heads * sp.vdim,) + (
        (sp.heads * sp.dim, sp.heads * sp.vdim) if sp.general else (sp.heads, sp.rank_g)) + (sp.rank_w,)
    assert all(0 <= o and o + n <= x.shape[1] for o, n in zip(sp.at, ends))
    if sp.general:
        assert wt.ab.numel() == wt.gain.numel() == sp.heads * sp.dim and sp.dim == sp.vdim and sp.heads == sp.kv_heads
    else:
        assert wt.ab.numel() == sp.heads and wt.gain.numel() == sp.vdim and sp.taps >= 1
        assert wt.conv.shape == (sp.conv_channels, sp.taps) and wt.lo_g.shape == (sp.heads * sp.vdim, sp.rank_g)
        assert ring.is_contiguous() and ring.dtype == torch.float32 and ring.shape[1] == sp.taps * sp.conv_channels
    assert all(t.dtype == torch.int32 and t.shape[0] >= x.shape[0] for t in (pos, slots))
    a = _Args()
    if code is None:
        return a, None
    if _lib.require().kca_delta_abi() != ctypes.sizeof(_Args):
        raise RuntimeError("kca_delta descriptor: C and ctypes sizes differ")
    a.x, a.ld = x.data_ptr(), x.stride(0)
    a.o_q, a.o_k, a.o_v, a.o_a, a.o_g, a.o_w = sp.at
    a.H, a.G, a.dk, a.dv, a.taps, a.rank_w, a.rank_g = (sp.heads, sp.kv_heads, sp.dim, sp.vdim, sp.taps, sp.rank_w,
                                                        sp.rank_g)
    p = _lib.ptr
    a.lo_w, a.lo_g, a.w0, a.ab, a.conv, a.gain = (p(wt.lo_w), p(wt.lo_g), p(wt.w0), p(wt.ab), p(wt.conv), p(wt.gain))
    a.eps, a.qscale = sp.eps, sp.dim ** -0.5
    a.state, a.ring = p(state), p(ring)
    a.pos, a.slot = p(pos), p(slots)
    a.out, a.ldo = p(out), out.stride(0)
    return a, code


def _call(name, a, *args):
    fn = getattr(_lib.require(), name)
    fn.argtypes = [ctypes.c_void_p] + [ctypes.c_int] * len(args) + [ctypes.c_void_p]
    fn.restype = ctypes.c_int
    rc = fn(ctypes.addressof(a), *args, _lib.stream())
    if rc != 0:
        raise RuntimeError(f"{name} returned status {rc} (unsupported shape/arguments)")
    _lib.LAUNCHES[0] += 1
    if _lib.SYNC_LAUNCH:
        torch.cuda.synchronize()


def delta_step(sp: DeltaHeads, wt: DeltaWeights, x, state, ring, pos, slots, out) -> torch.Tensor:
    """One token per row: row b continues ``slots[b]`` at ``pos[b]``."""
    a, code = _args(sp, wt, x, state, ring, pos, slots, out)
    if code is None:
        ent = [(i, 1, int(p), int(s)) for i, (p, s) in enumerate(zip(pos, slots))][:x.shape[0]]
        return _reference(sp, wt, x, state, ring, ent, out, None, None)
    _call("kca_delta_step", a, code, 0 if sp.general else 1, x.shape[0])
    return out


def low_rank_inner(sp: DeltaHeads, x, tanh) -> tuple[torch.Tensor, torch.Tensor | None]:
    """Inputs of the second-step products of a batch: (decay, gate | None). ``tanh(src)`` -> new tensor."""
    w = x[:, sp.at[5]:sp.at[5] + sp.rank_w]
    return (tanh(w) if sp.general else w), (None if sp.general else x[:, sp.at[4]:sp.at[4] + sp.rank_g])


def delta_portions(sp: DeltaHeads, wt: DeltaWeights, x, state, ring, b: Portions, out, dw, dg) -> torch.Tensor:
    """Portions of any sizes. ``dw`` [T, H dk] / ``dg`` [T, H dv] (channel): the second-step products."""
    a, code = _args(sp, wt, x, state, ring, b.pos, b.slots, out)
    T = x.shape[0]
    if code is None:
        return _reference(sp, wt, x, state, ring, b.ent.tolist(), out, dw, dg)
    assert dw.stride(1) == 1 and dw.shape == (T, sp.heads * sp.dim) and dw.dtype == x.dtype
    a.dw, a.ldw = dw.data_ptr(), dw.stride(0)
    if not sp.general:
        assert dg.stride(1) == 1 and dg.shape == (T, sp.heads * sp.vdim) and dg.dtype == x.dtype
        a.dg, a.ldg = dg.data_ptr(), dg.stride(0)
    assert b.ent.dtype == torch.int32 and b.ent.is_contiguous() and all(t.dtype == torch.int32 for t in (b.e0, b.e1))
    a.e0, a.e1, a.ent = b.e0.data_ptr(), b.e1.data_ptr(), b.ent.data_ptr()
    kind = 0 if sp.general else 1
    per = -(-(5 * sp.dim + sp.vdim + 2) // 4) * 4
    pk = torch.empty(T * sp.heads * per, device=x.device, dtype=torch.float32)
    o = torch.empty(T, sp.heads * sp.vdim, device=x.device, dtype=torch.float32)
    a.pk, a.o = pk.data_ptr(), o.data_ptr()
    _call("kca_delta_prep", a, code, kind, T)
    _call("kca_delta_scan", a, b.ent.shape[0])
    _call("kca_delta_gate", a, code, kind, T)
    return out


def _reference(sp, wt, x, state, ring, entries, out, dw, dg):
    H, G, D, E, n = sp.heads, sp.kv_heads, sp.dim, sp.vdim, sp.taps
    xf = x.float()
    col = lambda i, w: xf[:, sp.at[i]:sp.at[i] + w]  # noqa: E731
    if dw is None:
        inner = torch.tanh(col(5, sp.rank_w)) if sp.general else col(5, sp.rank_w)
        dw = inner @ wt.lo_w.float().t()
    lw = (dw.float() + wt.w0.float()).view(-1, H, D)
    if sp.general:
        q, k, v = (col(i, H * D).reshape(-1, H, D) for i in range(3))
        w = torch.exp(-math.exp(-0.5) * torch.sigmoid(lw))
        u = k * torch.rsqrt((k * k).sum(-1, keepdim=True) + 1e-6)
        z, p = u, -u * torch.sigmoid(col(3, H * D) + wt.ab.float()).view(-1, H, D)
        gate = torch.sigmoid(col(4, H * E)).view(-1, H, E)
    else:
        raw = torch.cat([col(0, G * D), col(1, G * D), col(2, H * E)], 1)
        cv, C = torch.empty_like(raw), raw.shape[1]
        taps = wt.conv.float()
        for r0, m, pos, slot in entries:
            rg = ring[slot].view(n, C)
            past = torch.stack([rg[(pos - i) % n] if pos - i >= 0 else torch.zeros(C) for i in range(n - 1, 0, -1)] or
                               [torch.zeros(C)])[:n - 1]
            seq = torch.cat([past, raw[r0:r0 + m]])
            for t in range(m):
                cv[r0 + t] = (seq[t:t + n] * taps.t()).sum(0)
            for t in range(max(0, m - n), m):
                rg[(pos + t) % n] = raw[r0 + t]
        cv = cv * torch.sigmoid(cv)
        unit = lambda y: y * torch.rsqrt((y * y).sum(-1, keepdim=True) + 1e-6)  # noqa: E731
        q = unit(cv[:, :G * D].view(-1, G, D)).repeat_interleave(H // G, 1) * D ** -0.5
        u = unit(cv[:, G * D:2 * G * D].view(-1, G, D)).repeat_interleave(H // G, 1)
        v = cv[:, 2 * G * D:].view(-1, H, E)
        w = torch.exp(-torch.exp(wt.ab.float())[:, None] * torch.nn.functional.softplus(lw))
        k = u * torch.sigmoid(col(3, H))[..., None]
        z, p = w * u, -k
        if dg is None:
            dg = col(4, sp.rank_g) @ wt.lo_g.float().t()
        gate = torch.sigmoid(dg.float()).view(-1, H, E)
    gain = wt.gain.float().view(H, E) if sp.general else wt.gain.float()
    for r0, m, pos, slot in entries:
        S = state[slot].view(H, D, E).clone() if pos > 0 else torch.zeros(H, D, E)
        for t in range(r0, r0 + m):
            s = (z[t][:, None] @ S)
            S = w[t][..., None] * S + p[t][..., None] * s + k[t][..., None] * v[t][:, None]
            o = (q[t][:, None] @ S)[:, 0]
            o = o * torch.rsqrt((o * o).mean(-1, keepdim=True) + sp.eps) * gain * gate[t]
            out[t] = o.reshape(-1).to(out.dtype)
        state[slot] = S.reshape(-1)
    return out


__all__ = ["DeltaHeads", "DeltaWeights", "Portions", "delta_step", "delta_portions", "low_rank_inner"]
