"""One decoded token per row through windowed attention over block means and a matrix memory in one launch
(``csrc/kernels/side_step.hip``): both read column blocks of the same projection rows, and neither fills the chip alone.
"""
from __future__ import annotations

import ctypes

import torch

from . import _lib
from . import biased_attention as ba
from . import matrix_memory as mm
from . import pooled_attention as pa


class _Args(ctypes.Structure):
    _fields_ = [("a", ba._Args), ("m", mm._Args), ("rows", ctypes.c_int), ("na", ctypes.c_int)]


def step_ok(sp: pa.PooledHeads, ms: mm.MemoryHeads, x: torch.Tensor) -> bool:
    """Sizes the common launch takes (``x``: the attention's projection columns)."""
    return (x.is_cuda and x.dtype == torch.bfloat16 and sp.heads > sp.kv_heads and sp.dim % 8 == 0 and sp.vdim % 8 == 0
            and sp.dim <= 128 and sp.vdim <= 128 and 32 < ms.dim <= 128 and ms.vdim % 4 == 0
            and all(o % 8 == 0 for o in sp.at) and x.stride(0) % 8 == 0 and x.data_ptr() % 16 == 0)


def step(attn: tuple, mem: tuple, pos, slots, max_len: int, ws=None, cnt=None):
    """``attn``: (heads, weights, projection columns, cache, out) of ``pooled_attention.attend_rows``; ``mem``: (heads, weights,
    projection columns, state, out) of ``matrix_memory.memory_step``."""
    sp, wt, x, cache, out = attn
    a, n, wsn, cn, kv, keep = pa.rows_args(sp, wt, x, cache, pos, slots, out, max_len, True, None, ws, cnt)
    m, code = mm._args(*mem[:4], pos, slots, mem[4])
    assert code == 1 and mem[2].shape[0] == n
    lib = _lib.require()
    if lib.kca_side_step_abi() != ctypes.sizeof(_Args):
        raise RuntimeError("kca_side_step descriptor: C and ctypes sizes differ")
    fn = lib.kca_side_step
    fn.argtypes = [ctypes.c_void_p, ctypes.c_void_p, ctypes.c_int, ctypes.c_longlong, ctypes.c_longlong, ctypes.c_int, ctypes.c_void_p]
    fn.restype = ctypes.c_int
    _lib.call("kca_side_step", ctypes.addressof(a), ctypes.addressof(m), n, wsn, cn, kv, _lib.stream())
    del keep


__all__ = ["step", "step_ok"]
