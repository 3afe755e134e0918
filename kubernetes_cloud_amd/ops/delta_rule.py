"""Delta-rule token mixers over a flat batch of sequence portions (``csrc/kernels/delta_rule.h``).

Per head a state S [dk, dv] of a sequence follows

    S_t = diag(w_t) S_(t-1) + p_t (z_t^T S_(t-1)) + k_t v_t^T,     o_t = S_t^T q_t

and the read-out is RMS-normed per head, times a gain, times a sigmoid gate. Two forms make the vectors from
the projections ``x`` (column blocks named by ``DeltaHeads.at``):

* general: w = exp(-e^(-1/2) sigmoid(lw + w0)), z = u = k / sqrt(|k|^2 + 1e-6), p = -(a u), a = sigmoid(.. + b)
* channel: q, k, v through short causal convolutions and silu; unit q (times dk^(-1/2)) and k, shared by groups
  of heads; w = exp(-exp(A) softplus(lw + dt)), z = w k, p = -beta k, k <- beta k

lw is the second step of a two-step projection (general: tanh between).

* head: as channel, with one decay per head: w = exp(-exp(A) softplus(lw + dt)), lw a projection; gate silu(g)
* ssd (a selective state space): q, k, v are C, B, x through short convolutions (with a bias) and silu, C and B
  shared by groups of heads; with dt = softplus(lw + bias): w = exp(-exp(A) dt), k <- dt k, no correction (p = 0),
  o += D v; the heads' read-outs times silu(z) are RMS-normed in equal parts, times a gain

Vectors, state and gates are fp32.
The state of a sequence lives in row ``slot`` of ``state``; the convolution inputs of its last positions in
``ring`` (position p in row p % taps). Both count as zero at and before position 0.
"""
from __future__ import annotations

import ctypes
import dataclasses
import math

import numpy as np
import torch

from . import _lib
from .rms_shift import native_dt


_P, _LL, _I, _F = ctypes.c_void_p, ctypes.c_longlong, ctypes.c_int, ctypes.c_float


class _Args(ctypes.Structure):
    _fields_ = [("x", _P), ("ld", _LL), *[(n, _I) for n in ("o_q", "o_k", "o_v", "o_a", "o_g", "o_w")],
                *[(n, _I) for n in ("H", "G", "dk", "dv", "taps", "rank_w", "rank_g")], ("lo_w", _P), ("lo_g", _P),
                ("dw", _P), ("ldw", _LL), ("dg", _P), ("ldg", _LL), ("w0", _P), ("ab", _P), ("conv", _P), ("gain", _P),
                ("eps", _F), ("qscale", _F), ("state", _P), ("ring", _P), ("pos", _P), ("slot", _P), ("e0", _P),
                ("e1", _P), ("out", _P), ("ldo", _LL), ("rows", _P), ("pk", _P), ("o", _P), ("ent", _P),
                ("cx", _P), ("convb", _P), ("skip", _P), ("norm_groups", _I)]


class _ChunkArgs(ctypes.Structure):
    _fields_ = [("d", _Args), ("ck", _P), ("en", _P), ("m", _P), ("b", _P), ("q", _P), ("oo", _P), ("e", _P)]


class _SsdArgs(ctypes.Structure):
    _fields_ = [("d", _Args), ("ck", _P), ("en", _P), ("cb", _P), ("bt", _P), ("gd", _P)]


FORMS = {"channel": 1, "head": 2, "ssd": 3}
CHUNK = 64       # tokens of a matrix-core chunk
CHUNK_MIN = 16   # shorter portions go token by token


@dataclasses.dataclass(frozen=True)
class DeltaHeads:
    """Sizes and constants of one layer. ``at``: first column of q, k, v, a (removal or beta), g (gate or its
    first step) and w (the decay's first step; head, ssd: its logits) in the projection rows. ``form`` names the
    rule of a layer that is not general; ``norm_groups``: equal parts of ssd's closing norm."""
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
    form: str = "channel"
    norm_groups: int = 1

    @property
    def kind(self) -> int:
        return 0 if self.general else FORMS[self.form]

    @property
    def conv_channels(self) -> int:
        return 0 if self.general else 2 * self.kv_heads * self.dim + self.heads * self.vdim

    @property
    def state_width(self) -> int:
        return self.heads * self.dim * self.vdim


@dataclasses.dataclass(frozen=True)
class DeltaWeights:
    """``ab``: bias of a (general) or A per head (others); ``lo_w``: general and channel; ``lo_g``: channel;
    ``conv``: all but general; ``conv_b``, ``skip`` (D): ssd."""
    lo_w: torch.Tensor | None
    w0: torch.Tensor
    ab: torch.Tensor
    gain: torch.Tensor
    lo_g: torch.Tensor | None = None
    conv: torch.Tensor | None = None
    conv_b: torch.Tensor | None = None
    skip: torch.Tensor | None = None


@dataclasses.dataclass
class Portions:
    """Device arrays of a batch of portions (``plan_portions``): per row its position, slot, and the first and
    one-past-last row of its entry; ``ent`` [n, 5] every entry, ``short`` / ``rows`` the short entries and their
    token rows, ``chunked`` [n, 6] / ``chunks`` [n, 4] the longer entries and their chunks."""
    pos: torch.Tensor
    slots: torch.Tensor
    e0: torch.Tensor
    e1: torch.Tensor
    ent: torch.Tensor
    short: torch.Tensor
    rows: torch.Tensor
    chunked: torch.Tensor
    chunks: torch.Tensor


def plan_portions(entries) -> dict:
    """[(first row, rows, position, slot)] -> host arrays of ``Portions`` (pos and slots aside), int32."""
    n_of = [e[1] for e in entries]
    out = {"e0": np.repeat([e[0] for e in entries], n_of), "e1": np.repeat([e[0] + e[1] for e in entries], n_of)}
    ent, short, rows, chunked, chunks = [], [], [], [], []
    for r0, n, pos, slot in entries:
        ent.append((r0, n, pos, slot, r0))
        if n < CHUNK_MIN:
            short.append((r0, n, pos, slot, len(rows)))
            rows += range(r0, r0 + n)
        else:
            nc = -(-n // CHUNK)
            chunked.append((r0, n, pos, slot, len(chunks), nc))
            chunks += [(r0 + i * CHUNK, min(CHUNK, n - i * CHUNK), r0, pos + i * CHUNK) for i in range(nc)]
    for k, v, w in (("ent", ent, 5), ("short", short, 5), ("rows", rows, 0), ("chunked", chunked, 6), ("chunks", chunks, 4)):
        v = np.asarray(v, dtype=np.int32)
        out[k] = v.reshape(-1, w) if w else v
    return {k: v.astype(np.int32) for k, v in out.items()}


def chunks_ok(sp: DeltaHeads, dtype) -> bool:
    """Sizes the chunked matrix-core kernels take (others, and fp32, run token by token)."""
    return (dtype == torch.bfloat16 and sp.dim % 8 == 0 and sp.vdim % 8 == 0 and sp.dim <= 128
            and (sp.kind == 3 or sp.vdim <= 128) and (sp.kind != 1 or sp.taps <= 4))


def _args(sp: DeltaHeads, wt: DeltaWeights, x, state, ring, pos, slots, out) -> tuple[_Args, int]:
    params = (wt.lo_w, wt.w0, wt.ab, wt.gain, wt.lo_g, wt.conv, wt.conv_b, wt.skip)
    code = native_dt(x, *params, out)
    kind, H, HV = sp.kind, sp.heads, sp.heads * sp.vdim
    assert x.stride(1) == 1 and out.stride(1) == 1 and out.shape == (x.shape[0], HV)
    assert state.is_contiguous() and state.dtype == torch.float32 and state.shape[1] == sp.state_width
    assert all(t is None or t.is_contiguous() for t in params)
    third = {0: (H * sp.dim, HV, sp.rank_w), 1: (H, sp.rank_g, sp.rank_w), 2: (H, HV, H), 3: (0, HV, H)}[kind]
    ends = (sp.kv_heads * sp.dim,) * 2 + (HV,) + third
    assert all(0 <= o and o + n <= x.shape[1] for o, n in zip(sp.at, ends))
    if kind < 2:
        assert wt.lo_w.shape == (H * sp.dim, sp.rank_w) and wt.w0.numel() == H * sp.dim
    else:
        assert wt.lo_w is None and wt.w0.numel() == H and sp.rank_w == sp.rank_g == 0
    if sp.general:
        assert wt.ab.numel() == wt.gain.numel() == H * sp.dim and sp.dim == sp.vdim and H == sp.kv_heads
    else:
        assert wt.ab.numel() == H and wt.gain.numel() == (HV if kind == 3 else sp.vdim) and sp.taps >= 1
        assert wt.conv.shape == (sp.conv_channels, sp.taps) and (kind != 1 or wt.lo_g.shape == (HV, sp.rank_g))
        assert ring.is_contiguous() and ring.dtype == torch.float32 and ring.shape[1] == sp.taps * sp.conv_channels
        assert wt.conv_b is None or wt.conv_b.numel() == sp.conv_channels
        assert kind != 3 or (wt.skip.numel() == H and HV % sp.norm_groups == 0)
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
    a.eps, a.qscale, a.norm_groups = sp.eps, sp.dim ** -0.5, sp.norm_groups
    a.convb, a.skip = p(wt.conv_b), p(wt.skip)
    a.state, a.ring = p(state), p(ring)
    a.pos, a.slot = p(pos), p(slots)
    a.out, a.ldo = p(out), out.stride(0)
    return a, code


def _call(name, a, *args, ptrs=()):
    fn = getattr(_lib.require(), name)
    fn.argtypes = [ctypes.c_void_p] + [ctypes.c_int] * len(args) + [ctypes.c_void_p] * (len(ptrs) + 1)
    fn.restype = ctypes.c_int
    rc = fn(ctypes.addressof(a), *args, *ptrs, _lib.stream())
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
    if sp.kind == 3:
        o = torch.empty(x.shape[0], sp.heads * sp.vdim, device=x.device, dtype=x.dtype)
        a.o = o.data_ptr()
    _call("kca_delta_step", a, code, sp.kind, x.shape[0])
    if sp.kind == 3:
        _call("kca_delta_parts", a, code, x.shape[0])
    return out


def low_rank_inner(sp: DeltaHeads, x, tanh) -> tuple[torch.Tensor, torch.Tensor | None]:
    """Inputs of the second-step products of a batch (general, channel): (decay, gate | None). ``tanh(src)`` -> new
    tensor."""
    w = x[:, sp.at[5]:sp.at[5] + sp.rank_w]
    return (tanh(w) if sp.general else w), (None if sp.general else x[:, sp.at[4]:sp.at[4] + sp.rank_g])


def delta_portions(sp: DeltaHeads, wt: DeltaWeights, x, state, ring, b: Portions, out, dw=None, dg=None) -> torch.Tensor:
    """Portions of any sizes. ``dw`` [T, H dk] (general, channel) / ``dg`` [T, H dv] (channel): the second-step
    products."""
    a, code = _args(sp, wt, x, state, ring, b.pos, b.slots, out)
    T = x.shape[0]
    if code is None:
        return _reference(sp, wt, x, state, ring, b.ent[:, :4].tolist(), out, dw, dg)
    kind, dev, H = sp.kind, x.device, sp.heads
    if kind < 2:
        assert dw.stride(1) == 1 and dw.shape == (T, sp.heads * sp.dim) and dw.dtype == x.dtype
        a.dw, a.ldw = dw.data_ptr(), dw.stride(0)
    if kind == 1:
        assert dg.stride(1) == 1 and dg.shape == (T, sp.heads * sp.vdim) and dg.dtype == x.dtype
        a.dg, a.ldg = dg.data_ptr(), dg.stride(0)
    assert all(t.dtype == torch.int32 and t.is_contiguous() for t in (b.e0, b.e1, b.ent, b.short, b.rows, b.chunked, b.chunks))
    a.e0, a.e1 = b.e0.data_ptr(), b.e1.data_ptr()
    if kind >= 2:
        cx = torch.empty(T, sp.conv_channels, device=dev, dtype=x.dtype)
        _call("kca_delta_conv", a, code, kind, T, ptrs=(cx.data_ptr(),))
        a.cx = cx.data_ptr()
    o = torch.empty(T, H * sp.vdim, device=dev, dtype=x.dtype)
    a.o = o.data_ptr()
    chunked = chunks_ok(sp, x.dtype) and b.chunks.shape[0] > 0
    if chunked and kind == 3:
        nc, G, DK = b.chunks.shape[0], sp.kv_heads, (64 if sp.dim <= 64 else 128)
        cb, bt = (torch.empty(nc * G * n * CHUNK, device=dev, dtype=torch.bfloat16) for n in (CHUNK, DK))
        gd = torch.empty(nc * H * 2 * CHUNK, device=dev, dtype=torch.float32)
        if _lib.require().kca_ssd_chunk_abi() != ctypes.sizeof(_SsdArgs):
            raise RuntimeError("kca_ssd_chunk descriptor: C and ctypes sizes differ")
        c = _SsdArgs()
        c.d, c.ck, c.en = a, b.chunks.data_ptr(), b.chunked.data_ptr()
        c.cb, c.bt, c.gd = cb.data_ptr(), bt.data_ptr(), gd.data_ptr()
        _call("kca_ssd_chunks", c, nc, b.chunked.shape[0])
    elif chunked:
        nc, DK, DV = b.chunks.shape[0], (64 if sp.dim <= 64 else 128), (64 if sp.vdim <= 64 else 128)
        sizes = (DK * DK, DV * DK, CHUNK * DK, DV * CHUNK)
        ws = [torch.empty(nc * H * n, device=dev, dtype=torch.bfloat16) for n in sizes]
        e = torch.empty(nc * H * DK, device=dev, dtype=torch.float32)
        if _lib.require().kca_delta_chunk_abi() != ctypes.sizeof(_ChunkArgs):
            raise RuntimeError("kca_delta_chunk descriptor: C and ctypes sizes differ")
        c = _ChunkArgs()
        c.d, c.ck, c.en = a, b.chunks.data_ptr(), b.chunked.data_ptr()
        c.m, c.b, c.q, c.oo = (t.data_ptr() for t in ws)
        c.e = e.data_ptr()
        _call("kca_delta_map", c, kind, nc)
        _call("kca_delta_run", c, kind, b.chunked.shape[0])
    ent, rows = (b.short, b.rows) if chunked else (b.ent, None)
    if ent.shape[0]:
        n = T if rows is None else rows.shape[0]
        pk = torch.empty(n * H * (-(-(5 * sp.dim + sp.vdim + 2) // 4) * 4), device=dev, dtype=torch.float32)
        a.pk, a.rows, a.ent = pk.data_ptr(), _lib.ptr(rows), ent.data_ptr()
        _call("kca_delta_prep", a, code, kind, n)
        _call("kca_delta_scan", a, code, ent.shape[0])
    if kind == 3:
        _call("kca_delta_parts", a, code, T)
    else:
        _call("kca_delta_gate", a, code, kind, T)
    return out


def _convolved(sp, wt, raw, ring, entries):
    """silu of the short convolutions of ``raw`` [T, channels]; the entries' last inputs go into their rings."""
    n, cv, C = sp.taps, torch.empty_like(raw), raw.shape[1]
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
    if wt.conv_b is not None:
        cv = cv + wt.conv_b.float()
    return cv * torch.sigmoid(cv)


def _reference(sp, wt, x, state, ring, entries, out, dw, dg):
    H, G, D, E = sp.heads, sp.kv_heads, sp.dim, sp.vdim
    softplus = torch.nn.functional.softplus
    xf = x.float()
    col = lambda i, w: xf[:, sp.at[i]:sp.at[i] + w]  # noqa: E731
    unit = lambda y: y * torch.rsqrt((y * y).sum(-1, keepdim=True) + 1e-6)  # noqa: E731
    if sp.kind < 2:
        if dw is None:
            inner = torch.tanh(col(5, sp.rank_w)) if sp.general else col(5, sp.rank_w)
            dw = inner @ wt.lo_w.float().t()
        lw = (dw.float() + wt.w0.float()).view(-1, H, D)
    else:
        lw = (col(5, H) + wt.w0.float())[..., None]
    if sp.general:
        q, k, v = (col(i, H * D).reshape(-1, H, D) for i in range(3))
        w = torch.exp(-math.exp(-0.5) * torch.sigmoid(lw))
        u = k * torch.rsqrt((k * k).sum(-1, keepdim=True) + 1e-6)
        z, p = u, -u * torch.sigmoid(col(3, H * D) + wt.ab.float()).view(-1, H, D)
        gate = torch.sigmoid(col(4, H * E)).view(-1, H, E)
    else:
        cv = _convolved(sp, wt, torch.cat([col(0, G * D), col(1, G * D), col(2, H * E)], 1), ring, entries)
        q, k = (y.reshape(-1, G, D).repeat_interleave(H // G, 1) for y in (cv[:, :G * D], cv[:, G * D:2 * G * D]))
        v = cv[:, 2 * G * D:].view(-1, H, E)
        w = torch.exp(-torch.exp(wt.ab.float())[:, None] * softplus(lw)).expand(-1, -1, D)
        if sp.kind == 3:
            k = k * softplus(lw)
            z = p = torch.zeros_like(k)
        else:
            u = unit(k)
            q, k = unit(q) * D ** -0.5, u * torch.sigmoid(col(3, H))[..., None]
            z, p = w * u, -k
            if sp.kind == 1:
                if dg is None:
                    dg = col(4, sp.rank_g) @ wt.lo_g.float().t()
                gate = torch.sigmoid(dg.float()).view(-1, H, E)
            else:
                gate = torch.nn.functional.silu(col(4, H * E)).view(-1, H, E)
    o = torch.empty(x.shape[0], H, E)
    for r0, m, pos, slot in entries:
        S = state[slot].view(H, D, E).clone() if pos > 0 else torch.zeros(H, D, E)
        for t in range(r0, r0 + m):
            s = (z[t][:, None] @ S)
            S = w[t][..., None] * S + p[t][..., None] * s + k[t][..., None] * v[t][:, None]
            o[t] = (q[t][:, None] @ S)[:, 0]
        state[slot] = S.reshape(-1)
    rms = lambda y: y * torch.rsqrt((y * y).mean(-1, keepdim=True) + sp.eps)  # noqa: E731
    if sp.kind == 3:
        y = (o + wt.skip.float()[:, None] * v).reshape(x.shape[0], H * E) * torch.nn.functional.silu(col(4, H * E))
        y = rms(y.view(x.shape[0], sp.norm_groups, -1)).reshape(x.shape[0], H * E) * wt.gain.float()
    else:
        y = rms(o) * (wt.gain.float().view(H, E) if sp.general else wt.gain.float()) * gate
    out.copy_(y.reshape(x.shape[0], H * E))
    return out


__all__ = ["DeltaHeads", "DeltaWeights", "Portions", "plan_portions", "chunks_ok", "delta_step", "delta_portions",
           "low_rank_inner"]
