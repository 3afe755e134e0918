"""Causal attention with a bias by distance, a sink and an output gate over the paged cache
(``csrc/kernels/biased_attn.hip``).

    w_j = exp(N(q) . N(k_j) * scale + bias[h, min(pos - j, n - 1)])
    o = sum_j w_j v_j / (exp(sink_h) + sum_j w_j) * sigmoid(g)

N: RMS norm per head with a gain. Query heads share key / value heads in groups. The projections are column blocks
of one buffer (``BiasedHeads.at``); norms, bias, sink and gate are optional. Cache layout: K pages
[pages, G, PS, dim] (normed keys), V pages [pages, G, PS, vdim].
"""
from __future__ import annotations

import ctypes
import dataclasses
import math

import torch

from . import _lib
from .decode import decode_chunk, gather_kv
from .diff_attention import MAX_SPLITS
from .rms_shift import native_dt


class _Args(ctypes.Structure):
    _P, _LL, _I, _F = ctypes.c_void_p, ctypes.c_longlong, ctypes.c_int, ctypes.c_float
    _fields_ = [("x", _P), ("ld", _LL), ("o_q", _I), ("o_k", _I), ("o_v", _I), ("o_g", _I), ("kc", _P), ("vc", _P),
                ("k_sp", _LL), ("v_sp", _LL), ("table", _P), ("tstride", _I), ("shift", _I), ("pos", _P), ("slot", _P),
                ("out", _P), ("ldo", _LL), ("H", _I), ("G", _I), ("dim", _I), ("vdim", _I), ("scale", _F), ("eps", _F),
                ("qn", _P), ("kn", _P), ("bias", _P), ("nb", _I), ("sink", _P), ("append", _I), ("nsplit", _I),
                ("chunk", _I), ("ws", _P), ("cnt", _P), ("tiles", _P), ("row_of", _P),
                # windowed attention over block means (ops/pooled_attention.py)
                ("window", _I), ("pool", _I), ("per", _I), ("pool_mul", ctypes.c_uint), ("kb", _P), ("vb", _P),
                ("kb_sp", _LL), ("vb_sp", _LL), ("freq", _P), ("rot", _I), ("mul", _F)]


@dataclasses.dataclass(frozen=True)
class BiasedHeads:
    """Sizes and constants of one layer's attention. ``at``: first columns of q, k, v and g (g < 0: no gate)."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    eps: float
    at: tuple


@dataclasses.dataclass(frozen=True)
class BiasedWeights:
    """``q_norm`` / ``k_norm`` [dim] gains; ``bias`` fp32 [H, n] by distance, the last column for all beyond;
    ``sink`` fp32 [H]. Each may be None."""
    q_norm: torch.Tensor | None = None
    k_norm: torch.Tensor | None = None
    bias: torch.Tensor | None = None
    sink: torch.Tensor | None = None


def distance_bucket(n: int, rows: int, far: float) -> int:
    """Row of a bias table with ``rows`` rows for distance ``n``: one row each below rows / 2, then rows evenly
    spaced in ln(n) up to ``far``, the last one beyond."""
    half = rows / 2
    if n < half:
        return n
    return min(rows - 1, int(half + math.floor(math.log(n / half) / math.log(far / half) * (rows - half))))


def bias_by_distance(table: torch.Tensor, far: float) -> torch.Tensor:
    """[rows, H] table -> fp32 [H, n], column d the bias at distance d, up to the first distance of the last row."""
    rows = table.shape[0]
    idx = [0]
    while idx[-1] < rows - 1:
        idx.append(distance_bucket(len(idx), rows, far))
    return table.float()[torch.tensor(idx, device=table.device)].t().contiguous()


def tiles_ok(sp: BiasedHeads, dtype, page_size: int, ld: int, ldo: int) -> bool:
    """Shapes the matrix-core kernel takes (others run the rows kernel)."""
    return (dtype == torch.bfloat16 and sp.dim % 8 == 0 and sp.vdim % 8 == 0 and sp.dim <= 128 and sp.vdim <= 256
            and all(o % 8 == 0 or o < 0 for o in sp.at) and ld % 8 == 0 and page_size >= 32 and ldo % 4 == 0)


def _abi():
    fn = _lib.require().kca_biased_attn_abi
    if fn() != ctypes.sizeof(_Args):
        raise RuntimeError(f"kca_biased_attn descriptor: C {fn()} bytes, ctypes {ctypes.sizeof(_Args)}")


def _args(sp: BiasedHeads, wt: BiasedWeights, x, k_pages, v_pages, table, pos, slots, out=None) -> _Args:
    PS = k_pages.shape[2]
    H, G, D, E = sp.heads, sp.kv_heads, sp.dim, sp.vdim
    assert x.stride(1) == 1 and all(o < 0 or o + n <= x.shape[1] for o, n in zip(sp.at, (H * D, G * D, G * E, H * E)))
    assert min(sp.at[:3]) >= 0
    assert k_pages.is_contiguous() and k_pages.shape[1:] == (G, PS, D)
    assert v_pages.is_contiguous() and v_pages.shape[1:] == (G, PS, E)
    assert v_pages.shape[0] == k_pages.shape[0] and PS >= 16 and PS & (PS - 1) == 0
    assert table.dtype == torch.int32 and table.is_contiguous()
    assert pos.dtype == torch.int32 and slots.dtype == torch.int32 and pos.shape[0] >= x.shape[0]
    assert all(t is None or (t.is_contiguous() and t.numel() == D and t.dtype == x.dtype) for t in (wt.q_norm, wt.k_norm))
    assert wt.bias is None or (wt.bias.is_contiguous() and wt.bias.dtype == torch.float32 and wt.bias.shape[0] == H)
    assert wt.sink is None or (wt.sink.is_contiguous() and wt.sink.dtype == torch.float32 and wt.sink.numel() == H)
    a, p = _Args(), _lib.ptr
    a.x, a.ld = x.data_ptr(), x.stride(0)
    a.o_q, a.o_k, a.o_v, a.o_g = sp.at
    a.kc, a.vc, a.k_sp, a.v_sp = k_pages.data_ptr(), v_pages.data_ptr(), k_pages.stride(0), v_pages.stride(0)
    a.table, a.tstride, a.shift = table.data_ptr(), table.stride(0), PS.bit_length() - 1
    a.pos, a.slot = pos.data_ptr(), slots.data_ptr()
    if out is not None:
        assert out.stride(1) == 1 and out.shape == (x.shape[0], H * E)
        a.out, a.ldo = out.data_ptr(), out.stride(0)
    a.H, a.G, a.dim, a.vdim, a.scale, a.eps = H, G, D, E, sp.scale, sp.eps
    a.qn, a.kn, a.bias, a.sink = p(wt.q_norm), p(wt.k_norm), p(wt.bias), p(wt.sink)
    a.nb = 0 if wt.bias is None else wt.bias.shape[1]
    return a


def _call(name, a, *args):
    if name.startswith("kca_biased"):  # (the pooled entry points check theirs)
        _abi()
    fn = getattr(_lib.require(), name)
    kinds = [ctypes.c_longlong if i in (2, 3) and name.endswith("_rows") else ctypes.c_int for i in range(len(args))]
    fn.argtypes, fn.restype = [ctypes.c_void_p, *kinds, ctypes.c_void_p], ctypes.c_int
    _lib.call(name, ctypes.addressof(a), *args, _lib.stream())


def append(sp: BiasedHeads, wt: BiasedWeights, x, k_pages, v_pages, table, pos, slots):
    """K (normed) / V of every row of ``x`` into its page."""
    code = native_dt(x, k_pages, v_pages)
    if code is None:
        T, G, D, E, PS = x.shape[0], sp.kv_heads, sp.dim, sp.vdim, k_pages.shape[2]
        k = _norm(x[:, sp.at[1]:sp.at[1] + G * D].reshape(T, G, D).float(), wt.k_norm, sp.eps)
        pg = table.long()[slots.long()[:T], pos.long()[:T] // PS]
        k_pages[pg, :, pos.long()[:T] % PS] = k.to(x.dtype)
        v_pages[pg, :, pos.long()[:T] % PS] = x[:, sp.at[2]:sp.at[2] + G * E].reshape(T, G, E)
        return
    _call("kca_biased_append", _args(sp, wt, x, k_pages, v_pages, table, pos, slots), code, x.shape[0])


def rows_plan(sp: BiasedHeads, rows: int, max_kv: int, target: int = 0, least: int = 64) -> tuple[int, int, int, int]:
    """(splits, keys per split, workspace floats, counters) of the rows kernel: enough for either head grouping.
    ``target``: workgroups to aim for with splits of one size, of ``least`` keys or more (0: ``decode_chunk``'s choice)."""
    hg = sp.heads // sp.kv_heads
    rb = 4 if hg > 1 else 1
    sub = -(-hg // rb)
    if target:
        n = min(MAX_SPLITS, max(1, target // (rows * sp.kv_heads * sub)), -(-max_kv // least))
        chunk = -(-max_kv // (32 * n)) * 32
    else:
        chunk = max(decode_chunk(rows, sp.kv_heads * sub, max_kv), -(-max_kv // MAX_SPLITS))
    n = -(-max_kv // chunk)
    return n, chunk, (rows * sp.kv_heads * sub * rb * n * (sp.vdim + 2) if n > 1 else 0), rows * sp.heads


def attend_rows(sp: BiasedHeads, wt: BiasedWeights, x, k_pages, v_pages, table, pos, slots, out, max_kv: int, *,
                fused_append: bool, row_of: torch.Tensor | None = None, ws: torch.Tensor | None = None,
                cnt: torch.Tensor | None = None):
    """One query token per row, over the row's own keys [0, pos]. ``fused_append``: the row's k / v come from ``x``
    and are stored on the way (single-token entries only); else the pages hold them already. ``row_of``: only these
    rows."""
    code = native_dt(x, k_pages, v_pages, out)
    if code is None:
        if fused_append:
            append(sp, wt, x, k_pages, v_pages, table, pos, slots)
        return _reference(sp, wt, x, k_pages, v_pages, table, pos, slots, out,
                          range(x.shape[0]) if row_of is None else row_of.tolist())
    n = x.shape[0] if row_of is None else row_of.shape[0]
    splits, chunk, wsf, blocks = rows_plan(sp, n, max_kv)
    if splits > 1:
        if ws is None or ws.numel() < wsf:
            ws = torch.empty(wsf, device=x.device, dtype=torch.float32)
        if cnt is None or cnt.numel() < blocks:
            cnt = torch.zeros(blocks, device=x.device, dtype=torch.int32)
    a = _args(sp, wt, x, k_pages, v_pages, table, pos, slots, out)
    a.append, a.nsplit, a.chunk, a.row_of = int(fused_append), splits, chunk, _lib.ptr(row_of)
    a.ws, a.cnt = _lib.ptr(ws), _lib.ptr(cnt)
    assert row_of is None or row_of.dtype == torch.int32
    _call("kca_biased_rows", a, code, n, ws.numel() if ws is not None else 0, cnt.numel() if cnt is not None else 0, int(max_kv))
    return out


def attend_tiles(sp: BiasedHeads, wt: BiasedWeights, x, k_pages, v_pages, table, pos, slots, out, tiles: torch.Tensor):
    """Prompt portions (``diff_attention.plan_tiles``) on the matrix cores; their K / V are in the pages."""
    assert native_dt(x, k_pages, v_pages, out) == 1 and tiles.dtype == torch.int32 and tiles.is_contiguous()
    a = _args(sp, wt, x, k_pages, v_pages, table, pos, slots, out)
    a.tiles = tiles.data_ptr()
    _call("kca_biased_tiles", a, tiles.shape[0])
    return out


def _norm(x, gain, eps):
    return x if gain is None else x * torch.rsqrt((x * x).mean(-1, keepdim=True) + eps) * gain.float()


def _reference(sp, wt, x, k_pages, v_pages, table, pos, slots, out, rows):
    H, G, D, E = sp.heads, sp.kv_heads, sp.dim, sp.vdim
    for t in rows:
        p, s = int(pos[t]), int(slots[t])
        q = _norm(x[t, sp.at[0]:sp.at[0] + H * D].float().view(H, D), wt.q_norm, sp.eps).view(G, H // G, D)
        k = gather_kv(k_pages, s, p + 1, table).float()  # [G, n, D]
        v = gather_kv(v_pages, s, p + 1, table).float()
        w = (torch.matmul(q, k.transpose(-1, -2)) * sp.scale).view(H, p + 1)
        if wt.bias is not None:
            w = w + wt.bias[:, (p - torch.arange(p + 1)).clamp(max=wt.bias.shape[1] - 1)]
        if wt.sink is not None:
            w = torch.cat([w, wt.sink[:, None]], 1)
        w = torch.softmax(w, -1)[:, :p + 1].view(G, H // G, p + 1)
        o = torch.matmul(w, v).reshape(H * E)
        if sp.at[3] >= 0:
            o = o * torch.sigmoid(x[t, sp.at[3]:sp.at[3] + H * E].float())
        out[t] = o.to(out.dtype)
    return out


__all__ = ["BiasedHeads", "BiasedWeights", "append", "attend_rows", "attend_tiles", "bias_by_distance",
           "distance_bucket", "rows_plan", "tiles_ok"]
