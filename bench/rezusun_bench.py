#!/usr/bin/env python3
"""Rezusun prefill / decode throughput beside Megusun (the framework's closest model: layers mixed of attention
and recurrences on the same runner) and GPT-J of equal size, and each kernel's distance from its roofline beside
the like kernel of those models (bench/megusun_bench.py).

Random weights. At every size the models have the same width, vocabulary and layer count, and about the same
weight bytes. Rezusun runs channel delta, general delta, latent attention, channel delta over and over, with a
gated feed-forward behind each. Through ``bench.py --rezusun`` or alone:

    python bench/rezusun_bench.py [--sizes ...] [--kernels]
"""
from __future__ import annotations

import argparse
import json
import os
import sys

sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

import torch

from megusun_bench import BF16_TFLOPS, HBM_TBPS, _runs, _time, gptj_cfg, megusun_cfg

# name -> (width, GPT-J heads, layers, vocab, head count at size 128, query latent, feed-forward)
SIZES = {"4096x8": (4096, 16, 8, 50400, 32, 1536, 10752), "2048x12": (2048, 16, 12, 50400, 16, 768, 5376)}
KV_RANK, ROT = 512, 64


def rezusun_cfg(d, heads, layers, vocab, q_rank, ff):
    mix = {"channel_delta": {"heads": heads, "kv_heads": heads, "dim": 128, "vdim": 128, "conv": 4, "decay_rank": 128,
                             "gate_rank": 128},
           "general_delta": {"heads": heads, "dim": 128, "decay_rank": 128},
           "latent_attention": {"heads": heads, "dim": 128, "rot_dim": ROT, "vdim": 128, "q_rank": q_rank,
                                "kv_rank": KV_RANK, "scale": (128 + ROT) ** -0.5, "rot": {"base": 1e4, "dims": ROT}}}
    order = ("channel_delta", "general_delta", "latent_attention", "channel_delta")
    return {"architecture": "Rezusun", "width": d, "vocab": vocab, "norm": {"eps": 1e-5},
            "layers": [{"type": order[i % 4], "mixer": mix[order[i % 4]], "mlp": {"kind": "dense", "ff": ff}}
                       for i in range(layers)]}


def run_models(sizes=None, batches=(1, 8, 32), prompt=1024, new_tokens=48, prefills=((1, 2048), (4, 2048)), only=None):
    from kubernetes_cloud_amd.models.causal_lm import build_model
    from kubernetes_cloud_amd.models.config import LMConfig
    dev = torch.device("cuda", torch.cuda.current_device())
    res = []
    for name in sizes or SIZES:
        d, gh, layers, vocab, heads, q_rank, ff = SIZES[name]
        for kind, cfg in (("gptj", gptj_cfg(d, gh, layers, vocab)), ("megusun", megusun_cfg(d, gh, layers, vocab)),
                          ("rezusun", rezusun_cfg(d, heads, layers, vocab, q_rank, ff))):
            if only and kind not in only:
                continue
            m = build_model(LMConfig.from_hf(cfg), device=dev, dtype=torch.bfloat16, seed=0).eval()
            r = {"size": name, "model": kind, "params_m": round(m.num_parameters() / 1e6),
                 **_runs(m, vocab, prompt, batches, new_tokens, prefills)}
            res.append(r)
            print("[rezusun_bench] " + json.dumps(r), file=sys.stderr, flush=True)
            del m
            torch.cuda.empty_cache()
    return res


def run_kernels(d=4096, heads=32, q_rank=1536, ff=10752, T=4096, cached=2048, batches=(1, 8, 32), ring=4):
    """[{kernel, us, roofline_us, share}] -- ``share`` = roofline time / measured time (operands cold in L2);
    ``like`` names the closest model's kernel, measured by ``megusun_bench.run_kernels`` on the same sizes."""
    import torch.nn.functional as F

    from kubernetes_cloud_amd.ops import delta_rule as dr
    from kubernetes_cloud_amd.ops import latent_attention as la
    from kubernetes_cloud_amd.ops import moe
    from kubernetes_cloud_amd.ops.norm_residual import NormedBranch, norm_residual
    dev = torch.device("cuda", torch.cuda.current_device())
    bf = dict(device=dev, dtype=torch.bfloat16)
    i32 = dict(device=dev, dtype=torch.int32)
    R, D, out = range(ring), 128, []

    def rec(kernel, us, bytes_=0.0, flops=0.0, like=None):
        roof = max(bytes_ / HBM_TBPS / 1e6, flops / BF16_TFLOPS / 1e6)
        r = {"kernel": kernel, "us": round(us, 2), "roofline_us": round(roof, 2), "share": round(roof / us, 3), "like": like}
        out.append(r)
        print("[rezusun_bench] " + json.dumps(r), file=sys.stderr, flush=True)

    # ---- norms and activation
    for n in (T, 32, 8, 1):
        xs, br = [torch.randn(n, d, device=dev) for _ in R], [torch.randn(n, d, **bf) for _ in R]
        w = torch.ones(d, **bf)
        us = _time([lambda x=x, b=b: norm_residual(x, NormedBranch(b, w, w, w), w, 1e-5) for x, b in zip(xs, br)])
        rec(f"norm_residual T={n}", us, n * d * 12, like="rms_shift")
    u, y, bu = [torch.randn(T, 2 * ff, **bf) for _ in R], torch.empty(T, ff, **bf), torch.zeros(2 * ff, **bf)
    us = _time([lambda x=x: moe.act_rows(x, y, True, act="gelu_tanh_gated", bias=bu) for x in u])
    rec(f"act_rows gated gelu T={T}", us, T * ff * 6, like="act_rows gelu")
    del u, y
    # ---- delta rule
    H, HD = heads, heads * D
    rank = 128

    def layer(general, seed=0):
        names = (("r", HD), ("k", HD), ("v", HD), ("g", HD), ("a", HD), ("w1", rank)) if general else \
            (("q", HD), ("k", HD), ("v", HD), ("a1", rank), ("g1", rank), ("b", H))
        at, o = {}, 0
        for n, c in names:
            at[n], o = o, o + c
        r = lambda *s, m=0.02: torch.randn(*s, **bf) * m  # noqa: E731
        if general:
            sp = dr.DeltaHeads(True, H, H, D, D, tuple(at[n] for n in ("r", "k", "v", "a", "g", "w1")), rank, 1e-5)
            wt = dr.DeltaWeights(r(HD, rank), r(HD), r(HD), r(HD))
        else:
            sp = dr.DeltaHeads(False, H, H, D, D, tuple(at[n] for n in ("q", "k", "v", "b", "g1", "a1")), rank, 1e-5, 4, rank)
            wt = dr.DeltaWeights(r(HD, rank), r(HD), r(H), r(D), r(HD, rank), r(sp.conv_channels, 4))
        return sp, wt, o

    for general in (True, False):
        sp, wt, cols = layer(general)
        kind = "general" if general else "channel"
        for n_seq in (1, 4):
            L = T // n_seq
            ent = [(i * L, L, 0, i) for i in range(n_seq)]
            pos, slots = torch.arange(L, **i32).repeat(n_seq), torch.arange(n_seq, **i32).repeat_interleave(L)
            pl = dr.Portions(pos, slots, **{k: torch.from_numpy(v).to(dev) for k, v in dr.plan_portions(ent).items()})
            xs = [torch.randn(T, cols, **bf) for _ in R]
            st = torch.zeros(n_seq, sp.state_width, device=dev)
            rg = None if general else torch.zeros(n_seq, 4 * sp.conv_channels, device=dev)
            dw, dg, o = torch.randn(T, HD, **bf), torch.randn(T, HD, **bf), torch.empty(T, HD, **bf)
            us = _time([lambda x=x: dr.delta_portions(sp, wt, x, st, rg, pl, o, dw, None if general else dg) for x in xs])
            rec(f"delta {kind} T={T} in {n_seq}", us, T * HD * 2 * (7 if general else 6) + n_seq * HD * D * 4, like="gated_scan")
        for B in batches:
            sts = [torch.zeros(B, sp.state_width, device=dev) for _ in range(max(2, min(8, 320 // (2 * B))))]
            rgs = [None if general else torch.zeros(B, 4 * sp.conv_channels, device=dev) for _ in sts]
            x, o = torch.randn(B, cols, **bf), torch.empty(B, HD, **bf)
            pos, slots = torch.full((B,), 9, **i32), torch.arange(B, **i32)
            us = _time([lambda s=s, r=r: dr.delta_step(sp, wt, x, s, r, pos, slots, o) for s, r in zip(sts, rgs)])
            low = (1 if general else 2) * HD * rank * 2
            rec(f"delta_step {kind} B={B}", us, B * (HD * D * 8 + cols * 2 + HD * 2) + low, like="gated_step")
    # ---- latent attention
    C, row = KV_RANK, KV_RANK + ROT
    sp = la.LatentHeads(H, D, ROT, D, q_rank, C, 192 ** -0.5, 1e-5, 1e4, ROT, (0, q_rank))
    r = lambda *s: torch.randn(*s, **bf) * 0.05  # noqa: E731
    ukv = r(H * 2 * D, C)
    wt = la.LatentWeights(r(q_rank), r(C), r(H), ukv[:HD].view(H, D, C).transpose(1, 2).contiguous(), ukv[HD:].view(H, D, C),
                          sp.frequencies().to(dev))
    for n_seq in (1, 4):
        L = T // n_seq
        ent = [(i * L, L, 0, i) for i in range(n_seq)]
        pages = torch.randn(T // 64 + 1, 1, 64, row, **bf)
        tbl = torch.arange(T // 64, **i32).view(n_seq, -1).contiguous()
        pos, slots = torch.arange(L, **i32).repeat(n_seq), torch.arange(n_seq, **i32).repeat_interleave(L)
        arr, num = la.plan_prompts(ent)
        pr = la.Prompts(**{k: torch.from_numpy(v).to(dev) for k, v in arr.items()}, **num)
        xs = [torch.randn(T, q_rank + row, **bf) for _ in R]
        if n_seq == 1:
            us = _time([lambda x=x: la.latent_append(sp, wt, x, pages, tbl, pos, slots) for x in xs])
            rec(f"latent_prep T={T}", us, T * (q_rank + row) * 4, like="rms_shift")
        q, o = torch.randn(T, H * (D + ROT), **bf), torch.empty(T, HD, **bf)
        kv = torch.randn(T, H * 2 * D, **bf)
        fl = n_seq * (L * L / 2) * H * 2 * (D + ROT + D)
        us = _time([lambda: la.attend_prompts(sp, wt, q, pages, tbl, pos, slots, o, ukv, pr, lambda a, b: kv)] * 2)
        rec(f"latent_tile {n_seq}x{L} H={H} (with gather)", us, 0, fl, like="diff_tile")
    for B in batches:
        nb = cached // 64
        n = max(2, min(8, int(1e9 / (B * cached * row * 2))))
        ps = [torch.randn(B * nb + 1, 1, 64, row, **bf) for _ in range(n)]
        tbl = torch.arange(B * nb, **i32).view(B, nb).contiguous()
        pos, slots = torch.full((B,), cached - 1, **i32), torch.arange(B, **i32)
        q, o = torch.randn(B, H * (D + ROT), **bf), torch.empty(B, HD, **bf)
        part = torch.empty(la.rows_plan(sp, B, cached)[2], device=dev)
        us = _time([lambda p=p: la.attend_rows(sp, wt, q, p, tbl, pos, slots, o, cached, part=part) for p in ps])
        rec(f"latent decode B={B} cached={cached} H={H} (3 launches)", us, B * cached * row * 2 + 2 * HD * C * 2,
            B * (cached * H * 2 * (row + C) + 4 * HD * C), like="diff_rows")
        del ps
    return out


def main():
    ap = argparse.ArgumentParser()
    ap.add_argument("--sizes", default="")
    ap.add_argument("--models", default="", help="gptj, megusun, rezusun")
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
