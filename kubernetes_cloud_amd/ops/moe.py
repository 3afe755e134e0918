"""Mixture of gated experts (``csrc/kernels/moe.hip``): top-k router (sigmoid scores, or softmax scores with a correction
of the choice, expert groups and identity experts), grouping by expert, expert products with the router weight on the
expert's input (or output), and the strided feed-forward activations (``csrc/kernels/act_rows.hip``).

Expert weights are stacked: gate-and-up [E, 2F, d] (gate rows first), down [E, d, F].
"""
from __future__ import annotations

import dataclasses
import math

import torch

from . import _lib
from .rms_shift import native_dt

GEMM_ROWS = 128
SHARED_ROWS = 16  # tokens up to which a shared expert's weights stream beside the routed ones'


@dataclasses.dataclass(frozen=True)
class Router:
    """How scores become choices. sigmoid: the ``top`` largest scores, which are the weights. softmax: the largest
    scores + ``correction`` (fp32 [outputs]) within the ``keep`` of ``groups`` equal groups of neighbours whose best one is
    largest; the weights are the scores over their sum. The last ``identity`` router outputs have no expert: they
    pass the token on."""
    softmax: bool = False
    correction: torch.Tensor | None = None
    groups: int = 1
    keep: int = 1
    identity: int = 0


SIGMOID = Router()


def route(h: torch.Tensor, router: torch.Tensor, top: int, shared_gate: torch.Tensor | None = None,
          rule: Router = SIGMOID):
    """h [T, d] -> (ids int32 [T, top], weights fp32 [T, top], sigmoid of the shared expert's gate [T] | None)."""
    code = native_dt(h, router, shared_gate)
    T, d = h.shape
    E = router.shape[0]
    if code is None:
        z = h.float() @ router.float().t()
        sg = torch.sigmoid(h.float() @ shared_gate.float().reshape(-1)) if shared_gate is not None else None
        if rule.softmax:
            s = torch.softmax(z, -1)
            c = s if rule.correction is None else s + rule.correction
            best = c.view(T, rule.groups, -1).amax(-1)
            kept = torch.zeros_like(best, dtype=torch.bool).scatter_(1, best.topk(rule.keep, dim=-1).indices, True)
            ids = c.masked_fill(~kept.repeat_interleave(E // rule.groups, 1), -torch.inf).topk(top, dim=-1).indices
            w = s.gather(1, ids)
            w = w / (w.sum(-1, keepdim=True) + 1e-20)
        else:
            w, ids = torch.sigmoid(z).topk(top, dim=-1)
        return ids.to(torch.int32), w, sg
    assert h.is_contiguous() and router.is_contiguous() and router.shape[1] == d
    ids = torch.empty(T, top, device=h.device, dtype=torch.int32)
    w = torch.empty(T, top, device=h.device, dtype=torch.float32)
    sg = torch.empty(T, device=h.device, dtype=torch.float32) if shared_gate is not None else None
    _lib.call("kca_moe_route", code, h.data_ptr(), router.data_ptr(), _lib.ptr(shared_gate), ids.data_ptr(),
              w.data_ptr(), _lib.ptr(sg), T, d, E, top, *_rule_args(rule, E), _lib.stream())
    return ids, w, sg


def _rule_args(rule: Router, E: int) -> tuple:
    c = rule.correction
    assert c is None or (c.is_contiguous() and c.dtype == torch.float32 and c.numel() == E and rule.softmax)
    return int(rule.softmax), _lib.ptr(c), rule.groups, rule.keep


@dataclasses.dataclass
class Groups:
    """Assignments sorted by expert, in tiles of at most ``mt`` rows of one expert."""
    perm: torch.Tensor
    inv: torch.Tensor     # [T, top]; -1: an identity expert
    tiles: torch.Tensor
    ntiles: torch.Tensor
    mt: int


def tile_rows(T: int, top: int, E: int, d: int, F: int, dtype) -> int:
    """Row limit of an expert tile: the matrix-core product (128) once an active expert expects enough rows
    to be worth a tile, else a streaming product of 1 .. 8 rows."""
    gemm = dtype == torch.bfloat16 and d % 8 == 0 and F % 8 == 0
    if gemm and T * top > 16 * min(E, T * top):
        return GEMM_ROWS
    return 1 if T == 1 else 2 if T == 2 else 4 if T <= 4 else 8


def _groups(T: int, top: int, E: int, mt: int, device) -> Groups:
    n = T * top
    z = dict(device=device, dtype=torch.int32)
    return Groups(torch.empty(n, **z), torch.empty(T, top, **z), torch.empty(min(E, n) + n // mt, 5, **z),
                  torch.empty(1, **z), mt)


def route_group(h: torch.Tensor, router: torch.Tensor, top: int, shared_gate: torch.Tensor | None, mt: int,
                rule: Router = SIGMOID):
    """``route`` and ``group`` -> (ids, weights, shared gate, groups); one launch for up to 16 bf16 tokens."""
    T, d = h.shape
    E = router.shape[0]
    real = E - rule.identity
    if native_dt(h, router, shared_gate) == 1 and T <= 16 and top <= 64 and d % 8 == 0 and (not rule.softmax or E <= 384):
        g = _groups(T, top, real, mt, h.device)
        ids = torch.empty(T, top, device=h.device, dtype=torch.int32)
        w = torch.empty(T, top, device=h.device, dtype=torch.float32)
        sg = torch.empty(T, device=h.device, dtype=torch.float32) if shared_gate is not None else None
        assert h.is_contiguous() and router.is_contiguous() and router.shape[1] == d
        _lib.call("kca_moe_route_group", h.data_ptr(), router.data_ptr(), _lib.ptr(shared_gate), ids.data_ptr(),
                  w.data_ptr(), _lib.ptr(sg), T, d, E, real, top, *_rule_args(rule, E), mt, g.perm.data_ptr(), g.inv.data_ptr(),
                  g.tiles.data_ptr(), g.tiles.shape[0], g.ntiles.data_ptr(), _lib.stream())
        return ids, w, sg, g
    ids, w, sg = route(h, router, top, shared_gate, rule)
    return ids, w, sg, group(ids, real, mt)


def group(ids: torch.Tensor, E: int, mt: int) -> Groups:
    """Ids of ``E`` and beyond (identity experts) take no row."""
    T, top = ids.shape
    n = T * top
    g = _groups(T, top, E, mt, ids.device)
    mx = g.tiles.shape[0]
    if not ids.is_cuda:
        flat = ids.reshape(-1)
        real = int((flat < E).sum())
        order = torch.argsort(flat, stable=True)
        g.perm.copy_(order)
        g.inv.view(-1)[order] = torch.where(torch.arange(n) < real, torch.arange(n), -1).to(torch.int32)
        g.perm[real:] = -1
        return g
    _lib.call("kca_moe_group", ids.data_ptr(), n, E, mt, g.perm.data_ptr(), g.inv.data_ptr(), g.tiles.data_ptr(), mx,
              g.ntiles.data_ptr(), _lib.stream())
    return g


def shared_ok(T: int, mt: int) -> bool:
    """Whether a shared expert streams beside the routed ones' (``experts``): few tokens, streaming products."""
    return mt != GEMM_ROWS and T <= SHARED_ROWS


def experts(h: torch.Tensor, ids: torch.Tensor, weights: torch.Tensor, gate_up: torch.Tensor, down: torch.Tensor,
            g: Groups, scale_in: bool = True, shared: tuple | None = None):
    """Output rows [n, d] of the routed experts in ``g``'s sorted order. ``shared`` (gate and up [2F', d], down [d, F']): an
    ungated expert for every token in the same launches (``shared_ok``) -> (rows, its output [T, d])."""
    E, F2, d = gate_up.shape
    F, top, n, T = F2 // 2, ids.shape[1], ids.numel(), h.shape[0]
    code = native_dt(h, gate_up, down, *(shared or ()))
    if code is None:
        flat, wt = ids.reshape(-1).long(), weights.reshape(-1)
        y = torch.empty(n, d, dtype=h.dtype)

        def ff(x, up, dn, s_in=1.0):
            u = up.float() @ (x * s_in)
            k = u.shape[0] // 2
            return dn.float() @ (torch.nn.functional.silu(u[:k]) * u[k:])

        for pos, a in enumerate(g.perm.tolist()):
            if a < 0:
                break
            e, w = int(flat[a]), float(wt[a])
            y[pos] = (ff(h[a // top].float(), gate_up[e], down[e], w if scale_in else 1.0) * (1.0 if scale_in else w)).to(h.dtype)
        return y if shared is None else (y, torch.stack([ff(r.float(), *shared).to(h.dtype) for r in h]))
    assert h.is_contiguous() and gate_up.is_contiguous() and down.is_contiguous() and down.shape == (E, d, F)
    act = torch.empty(n, F, device=h.device, dtype=h.dtype)
    y = torch.empty(n, d, device=h.device, dtype=h.dtype)
    mx = g.tiles.shape[0]
    common = (g.perm.data_ptr(), weights.data_ptr(), g.tiles.data_ptr(), g.ntiles.data_ptr(), mx, g.mt, top)
    up_s = down_s = (None, None, None, 0, 0, 0)
    if shared is not None:
        w_up, w_down = shared
        Fs = w_down.shape[1]
        assert shared_ok(T, g.mt) and w_up.is_contiguous() and w_down.is_contiguous() and w_up.shape == (2 * Fs, d)
        act_s, y_s = torch.empty(T, Fs, device=h.device, dtype=h.dtype), torch.empty(T, d, device=h.device, dtype=h.dtype)
        up_s = (h.data_ptr(), w_up.data_ptr(), act_s.data_ptr(), T, Fs, d)
        down_s = (act_s.data_ptr(), w_down.data_ptr(), y_s.data_ptr(), T, d, Fs)
    _lib.call("kca_moe_expert", code, h.data_ptr(), gate_up.data_ptr(), act.data_ptr(), *common, F, d, 1,
              int(scale_in), *up_s, _lib.stream())
    _lib.call("kca_moe_expert", code, act.data_ptr(), down.data_ptr(), y.data_ptr(), *common, d, F, 0,
              int(not scale_in), *down_s, _lib.stream())
    return y if shared is None else (y, y_s)


ACT_ROWS = {"gelu": 0, "silu_gated": 1, "gelu_tanh_gated": 2, "tanh": 3, "relu2": 4, "softcap": 5}


def act_rows(x: torch.Tensor, out: torch.Tensor, gated: bool, row_scale: torch.Tensor | None = None, *,
             act: str | None = None, bias: torch.Tensor | None = None, cap: float = 0.0) -> torch.Tensor:
    """out = gelu(x) (exact), or silu(gate) * up * row_scale with x = [gate | up]; strided rows. ``act`` names
    another form (``ACT_ROWS``; "softcap": cap tanh(x / cap)); ``bias`` is added to x first. Without a gate, out
    may be x."""
    T, F = out.shape
    act = act or ("silu_gated" if gated else "gelu")
    gated = act.endswith("_gated")
    code = native_dt(x, out, bias)
    assert x.shape == (T, 2 * F if gated else F) and x.stride(1) == 1 and out.stride(1) == 1
    assert bias is None or (bias.is_contiguous() and bias.numel() == x.shape[1])
    if code is None:
        xf = x.float() if bias is None else x.float() + bias.float()
        if gated:
            g = xf[:, :F]
            y = (torch.nn.functional.silu(g) if act == "silu_gated" else
                 0.5 * g * (1 + torch.tanh(math.sqrt(2 / math.pi) * (g + 0.044715 * g ** 3)))) * xf[:, F:]
            out.copy_(y if row_scale is None else y * row_scale[:, None])
        else:
            out.copy_(torch.tanh(xf) if act == "tanh" else torch.relu(xf) ** 2 if act == "relu2" else
                      cap * torch.tanh(xf / cap) if act == "softcap" else 0.5 * xf * (1 + torch.erf(xf / math.sqrt(2.0))))
        return out
    _lib.call("kca_act_rows", code, ACT_ROWS[act], x.data_ptr(), x.stride(0), _lib.ptr(row_scale), _lib.ptr(bias),
              out.data_ptr(), out.stride(0), T, F, float(cap), _lib.stream())
    return out


__all__ = ["Router", "SIGMOID", "route", "group", "route_group", "experts", "shared_ok", "act_rows", "tile_rows", "Groups"]
