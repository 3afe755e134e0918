#!/usr/bin/env python3
"""Gibipel prefill / decode throughput beside Begopel (two mixers side by side on the same runner) and Megusun with routed
experts at equal size, and each kernel's distance from its roofline beside the like kernel of those models
(bench/begopel_bench.py, bench/megusun_bench.py).

Random weights. At every size the models have the same width, vocabulary and layer count; Gibipel and the routed Megusun
have about the same weight bytes, and about the same per token. Through ``bench.py --gibipel`` or alone:

    python bench/gibipel_bench.py [--sizes ...] [--kernels]
"""
from __future__ import annotations

import argparse
import json
import os
import sys

sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

import torch

from begopel_bench import SIZES as BEGOPEL_SIZES, begopel_cfg
from megusun_bench import BF16_TFLOPS, HBM_TBPS, SIZES as MEGUSUN_SIZES, _runs, _time, megusun_cfg

# name -> (width, layers, vocab, attention heads of 128, its groups, memory heads of 128, experts, identity experts,
# groups of outputs, groups kept, top, expert ff, shared ff)
SIZES = {"4096x8": (4096, 8, 50400, 32, 8, 16, 16, 4, 4, 2, 3, 2048, 2048),
         "2048x12": (2048, 12, 50400, 16, 4, 8, 24, 8, 8, 4, 5, 768, 1024)}
D, WINDOW, POOL = 128, 1024, 16


def gibipel_cfg(d, layers, vocab, ah, ag, mh, experts, identity, groups, keep, top, ff, shared):
    rot = {"base": 500000.0, "dims": D, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}
    layer = {"type": "parallel", "mixer": {
        "left": {"heads": ah, "kv_heads": ag, "dim": D, "vdim": D, "scale": D ** -0.5, "mask": {"size": WINDOW, "pool": POOL}, "rot": rot},
        "right": {"heads": mh, "dim": D, "vdim": D, "gate_cap": 15.0}, "left_scale": 0.5, "right_scale": 0.5},
        "mlp": {"kind": "moe", "router": {"experts": experts, "identity": identity, "top": top, "groups": {"count": groups, "keep": keep}},
                "expert": {"ff": ff}, "shared": {"ff": shared}}}
    return {"architecture": "Gibipel", "width": d, "vocab": vocab, "norm": {"eps": 1e-5}, "embedding": {"scale": 1.0},
            "logit_scale": 1.0, "layers": [layer] * layers}


def run_models(sizes=None, batches=(1, 8, 32), prompt=1024, new_tokens=48, prefills=((1, 2048), (4, 2048)), only=None):
    from kubernetes_cloud_amd.models.causal_lm import build_model
    from kubernetes_cloud_amd.models.config import LMConfig
    dev = torch.device("cuda", torch.cuda.current_device())
    res = []
    for name in sizes or SIZES:
        d, layers, vocab = SIZES[name][:3]
        _, heads, _, _, moe = MEGUSUN_SIZES[name]
        for kind, cfg in (("begopel", begopel_cfg(*BEGOPEL_SIZES[name])),
                          ("megusun-moe", megusun_cfg(d, heads, layers, vocab, moe, kv_heads=heads // 4)),
                          ("gibipel", gibipel_cfg(*SIZES[name]))):
            if only and kind not in only:
                continue
            m = build_model(LMConfig.from_hf(cfg), device=dev, dtype=torch.bfloat16, seed=0).eval()
            r = {"size": name, "model": kind, "params_m": round(m.num_parameters() / 1e6),
                 **_runs(m, vocab, prompt, batches, new_tokens, prefills)}
            res.append(r)
            print("[gibipel_bench] " + json.dumps(r), file=sys.stderr, flush=True)
            del m
            torch.cuda.empty_cache()
    return res


def run_kernels(size="4096x8", T=4096, cached=2048, batches=(1, 8, 32), ring=4):
    """[{kernel, us, roofline_us, share}] -- ``share`` = roofline time / measured time (operands cold in L2); ``like``
    names the closest models' kernel, measured by ``begopel_bench`` / ``megusun_bench`` ``run_kernels``."""
    from kubernetes_cloud_amd.ops import delta_rule as dr
    from kubernetes_cloud_amd.ops import diff_attention as da
    from kubernetes_cloud_amd.ops import matrix_memory as mm
    from kubernetes_cloud_amd.ops import moe
    from kubernetes_cloud_amd.ops import pooled_attention as pa
    from kubernetes_cloud_amd.ops import side_step as ss
    from kubernetes_cloud_amd.ops.norm_residual import NormedSum, postnorm
    d, _, _, ah, ag, mh, E, ident, groups, keep, top, ff, _ = SIZES[size]
    dev = torch.device("cuda", torch.cuda.current_device())
    bf = dict(device=dev, dtype=torch.bfloat16)
    i32 = dict(device=dev, dtype=torch.int32)
    R, out = range(ring), []

    def rec(kernel, us, bytes_=0.0, flops=0.0, like=None):
        roof = max(bytes_ / HBM_TBPS / 1e6, flops / BF16_TFLOPS / 1e6)
        r = {"kernel": kernel, "us": round(us, 2), "roofline_us": round(roof, 2), "share": round(roof / us, 4), "like": like}
        out.append(r)
        print("[gibipel_bench] " + json.dumps(r), file=sys.stderr, flush=True)

    # ---- norms, alone and over routed rows
    one = torch.ones((), **bf)
    for n in (T, 32, 8, 1):
        xs, br = [torch.randn(n, d, device=dev) for _ in R], [torch.randn(n, d, **bf) for _ in R]
        us = _time([lambda x=x, b=b: postnorm(x, NormedSum(one, b), 1e-5, torch.bfloat16) for x, b in zip(xs, br)])
        rec(f"postnorm T={n}", us, n * d * 12, like="prenorm")
        ys = [torch.randn(n * top, d, **bf) for _ in R]
        inv, wts = torch.randperm(n * top, device=dev).view(n, top).to(torch.int32), torch.rand(n, top, device=dev)
        us = _time([lambda x=x, b=b, y=y: postnorm(x, NormedSum(one, b, y, inv, wts), 1e-5, torch.bfloat16) for x, b, y in zip(xs, br, ys)])
        rec(f"postnorm T={n} +{top} routed rows", us, n * d * (12 + 2 * top), like="rms_shift")
        del xs, br, ys

    # ---- router and experts
    rule = moe.Router(True, torch.zeros(E + ident, device=dev), groups, keep, ident)
    router = torch.randn(E + ident, d, **bf) * 0.02
    gu, dn = ([torch.randn(E, *s, **bf) * 0.02 for _ in range(2)] for s in ((2 * ff, d), (d, ff)))
    for n in (T, 32, 8, 1):
        hs = [torch.randn(n, d, **bf) for _ in R]
        mt = moe.tile_rows(n, top, E + ident, d, ff, torch.bfloat16)
        us = _time([lambda h=h: moe.route_group(h, router, top, None, mt, rule) for h in hs])
        rec(f"moe_route_group softmax T={n} E={E}+{ident}", us, n * d * 2 + (E + ident) * d * 2, like="moe_route_group")
        ids, w, _, g = moe.route_group(hs[0], router, top, None, mt, rule)
        real = int((ids < E).sum())
        used = ids[ids < E].unique().numel()
        us = _time([lambda a=a, b=b: moe.experts(hs[0], ids, w, a, b, g, False) for a, b in zip(gu, dn)])
        rec(f"moe_experts out-weighted T={n} E={E} rows={real} F={ff}", us, used * 3 * ff * d * 2 + (n * d + real * (d + 2 * ff)) * 2,
            real * 6 * d * ff, like="moe_experts")
    del gu, dn

    # ---- matrix memory
    V = mh * D
    sp = mm.MemoryHeads(mh, D, D, (0, V, 2 * V, 3 * V, 4 * V, 4 * V + 16), 15.0, 1e-5)
    cols = 4 * V + 32
    wt = mw = mm.MemoryWeights(torch.zeros(mh, **bf), torch.ones(mh, **bf) * 3, torch.ones(V, **bf))
    state = lambda n: mm.MemoryState(*(torch.zeros(n, w, device=dev) for w in (mh * D * D, mh * D, mh)))  # noqa: E731
    for n_seq in (1, 4):
        L = T // n_seq
        ent = [(i * L, L, 0, i) for i in range(n_seq)]
        pos, slots = torch.arange(L, **i32).repeat(n_seq), torch.arange(n_seq, **i32).repeat_interleave(L)
        pl = dr.Portions(pos, slots, **{k: torch.from_numpy(v).to(dev) for k, v in dr.plan_portions(ent).items()})
        xs, st, o = [torch.randn(T, cols, **bf) for _ in R], state(n_seq), torch.empty(T, V, **bf)
        us = _time([lambda x=x: mm.memory_portions(sp, wt, x, st, pl, o) for x in xs])
        rec(f"memory T={T} in {n_seq} H={mh}", us, T * (cols + V) * 2 + n_seq * mh * D * D * 4, like="delta ssd, delta head")
    for B in batches:
        sts = [state(B) for _ in range(max(2, min(8, 320 // B)))]
        x, o = torch.randn(B, cols, **bf), torch.empty(B, V, **bf)
        pos, slots = torch.full((B,), 9, **i32), torch.arange(B, **i32)
        us = _time([lambda s=s: mm.memory_step(sp, wt, x, s, pos, slots, o) for s in sts])
        rec(f"memory_step B={B} H={mh}", us, B * (mh * D * (D + 1) * 8 + cols * 2 + V * 2), like="delta_step head")

    # ---- windowed attention over block means
    AV, KV = ah * D, ag * D
    sp = pa.PooledHeads(ah, ag, D, D, D ** -0.5, 1e-5, (0, AV, AV + KV), WINDOW, POOL, D)
    wt = pa.PooledWeights(torch.ones(AV, **bf), torch.ones(KV, **bf), torch.zeros(ah, device=dev), pa.rotary_frequencies(D, 5e5).to(dev))
    cols, per = AV + 2 * KV, pa.block_rows(64, POOL)
    cache = lambda pages, tbl: pa.PooledCache(*(torch.randn(pages + 1, ag, n, D, **bf) for n in (64, 64, per, per)), tbl)  # noqa: E731
    for n_seq in (1, 4):
        L = T // n_seq
        c = cache(T // 64, torch.arange(T // 64, **i32).view(n_seq, -1).contiguous())
        pos, slot = torch.arange(L, **i32).repeat(n_seq), torch.arange(n_seq, **i32).repeat_interleave(L)
        tiles = torch.from_numpy(da.plan_tiles([(i * L, L, 0, i) for i in range(n_seq)])).to(dev)
        xs, o = [torch.randn(T, cols, **bf) for _ in range(2)], torch.empty(T, AV, **bf)
        if n_seq == 1:
            us = _time([lambda x=x: pa.prepare(sp, wt, x, c, pos, slot) for x in xs])
            rec(f"pooled_prep T={T} (2 launches)", us, T * cols * 4 + T * KV * 4 * (1 + 1 / POOL), like="biased_append, prenorm")
        us = _time([lambda x=x: pa.attend_tiles(sp, wt, x, c, pos, slot, o, tiles) for x in xs])
        seen = sum(sp.visible(i + 1) for i in range(L))
        rec(f"pooled_tile {n_seq}x{L} H={ah} G={ag}", us, 0, n_seq * seen * ah * 4 * D, like="biased_tile")
    for B in batches:
        nb = cached // 64
        n = max(2, min(8, int(1e9 / (B * cached * KV * 4))))
        cs = [cache(B * nb, torch.arange(B * nb, **i32).view(B, nb).contiguous()) for _ in range(n)]
        pos, slot = torch.full((B,), cached - 1, **i32), torch.arange(B, **i32)
        x, o, seen = torch.randn(B, cols, **bf), torch.empty(B, AV, **bf), sp.visible(cached)
        _, _, wsf, blk = pa.rows_plan(sp, B, seen)
        ws, cnt = torch.empty(max(wsf, 1), device=dev), torch.zeros(blk, **i32)
        us = _time([lambda c=c: pa.attend_rows(sp, wt, x, c, pos, slot, o, cached, fused=True, ws=ws, cnt=cnt) for c in cs])
        rec(f"pooled_rows B={B} cached={cached} seen={seen} H={ah} G={ag}", us, B * seen * KV * 4, like="biased_rows")
        ms = mm.MemoryHeads(mh, D, D, (0, V, 2 * V, 3 * V, 4 * V, 4 * V + 16), 15.0, 1e-5)
        xm, om, sts = torch.randn(B, 4 * V + 32, **bf), torch.empty(B, V, **bf), [state(B) for _ in cs]
        us = _time([lambda c=c, s=s: ss.step((sp, wt, x, c, o), (ms, mw, xm, s, om), pos, slot, cached, ws, cnt) for c, s in zip(cs, sts)])
        rec(f"side_step B={B} (pooled_rows and memory_step)", us, B * (seen * KV * 4 + mh * D * (D + 1) * 8), like="biased_rows, delta_step head")
        del cs, sts
    return out


def main():
    ap = argparse.ArgumentParser()
    ap.add_argument("--sizes", default="")
    ap.add_argument("--models", default="", help="begopel, megusun-moe, gibipel")
    ap.add_argument("--kernels", action="store_true", help="per-kernel rooflines instead of the models")
    ap.add_argument("--batches", default="1,8,32")
    ap.add_argument("--prompt", type=int, default=1024)
    ap.add_argument("--new-tokens", type=int, default=48)
    a = ap.parse_args()
    bs = tuple(int(x) for x in a.batches.split(","))
    if a.kernels:
        res = run_kernels(batches=bs)
    else:
        res = run_models(a.sizes.split(",") if a.sizes else None, bs, a.prompt, a.new_tokens,
                         only=a.models.split(",") if a.models else None)
    print(json.dumps(res))


if __name__ == "__main__":
    main()
