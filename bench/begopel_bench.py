#!/usr/bin/env python3
"""Begopel prefill / decode throughput beside Rezusun (the framework's closest model: delta rules and attention on the
same runner) and GPT-J of equal size, and each kernel's distance from its roofline beside the like kernel of those
models (bench/rezusun_bench.py, bench/megusun_bench.py).

Random weights. At every size the models have the same width, vocabulary and layer count, and about the same weight
bytes a layer. Begopel alternates state-space and side-by-side layers, with a squared-ReLU feed-forward behind each.
Through ``bench.py --begopel`` or alone:

    python bench/begopel_bench.py [--sizes ...] [--kernels]
"""
from __future__ import annotations

import argparse
import json
import os
import sys

sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

import torch

from megusun_bench import BF16_TFLOPS, HBM_TBPS, _runs, _time, gptj_cfg
from rezusun_bench import SIZES as REZUSUN_SIZES, rezusun_cfg

# name -> (width, layers, vocab, state-space heads of 64, its groups, attention heads of 128, its groups, delta heads
# of 128, its groups, feed-forward behind a state space, behind two mixers)
SIZES = {"4096x8": (4096, 8, 50400, 128, 8, 32, 8, 32, 16, 11264, 9216),
         "2048x12": (2048, 12, 50400, 64, 4, 16, 4, 16, 8, 5632, 4608)}
STATE, BIAS = 128, (32, 128)  # state size; rows and reach of the bias table


def begopel_cfg(d, layers, vocab, sh, sg, ah, ag, dh, dg, ff_s, ff_p, loop=None):
    ssd = {"type": "mamba2", "mixer": {"heads": sh, "groups": sg, "state": STATE, "vdim": 64, "conv": 4, "norm_groups": sg},
           "mlp": {"kind": "dense", "ff": ff_s}}
    pair = {"type": "parallel", "mixer": {
        "left": {"heads": ah, "kv_heads": ag, "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "bias_max": BIAS[1], "bias_rows": BIAS[0]},
        "right": {"heads": dh, "kv_heads": dg, "dim": 128, "vdim": 128, "conv": 4}}, "mlp": {"kind": "dense", "ff": ff_p}}
    cfg = {"architecture": "Begopel", "width": d, "vocab": vocab, "norm": {"eps": 1e-5}, "embedding": {"scale": 1.0},
           "logit_softcap": 30.0, "layers": [pair if i % 2 else ssd for i in range(layers)]}
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


def run_models(sizes=None, batches=(1, 8, 32), prompt=1024, new_tokens=48, prefills=((1, 2048), (4, 2048)), only=None):
    from kubernetes_cloud_amd.models.causal_lm import build_model
    from kubernetes_cloud_amd.models.config import LMConfig
    dev = torch.device("cuda", torch.cuda.current_device())
    res = []
    for name in sizes or SIZES:
        d, layers, vocab = SIZES[name][:3]
        _, gh, _, _, rh, q_rank, rff = REZUSUN_SIZES[name]
        for kind, cfg in (("gptj", gptj_cfg(d, gh, layers, vocab)), ("rezusun", rezusun_cfg(d, rh, layers, vocab, q_rank, rff)),
                          ("begopel", begopel_cfg(*SIZES[name]))):
            if only and kind not in only:
                continue
            m = build_model(LMConfig.from_hf(cfg), device=dev, dtype=torch.bfloat16, seed=0).eval()
            r = {"size": name, "model": kind, "params_m": round(m.num_parameters() / 1e6),
                 **_runs(m, vocab, prompt, batches, new_tokens, prefills)}
            res.append(r)
            print("[begopel_bench] " + json.dumps(r), file=sys.stderr, flush=True)
            del m
            torch.cuda.empty_cache()
    return res


def run_kernels(size="4096x8", T=4096, cached=2048, batches=(1, 8, 32), ring=4):
    """[{kernel, us, roofline_us, share}] -- ``share`` = roofline time / measured time (operands cold in L2); ``like``
    names the closest models' kernel, measured by ``rezusun_bench`` / ``megusun_bench`` ``run_kernels``."""
    from kubernetes_cloud_amd.ops import biased_attention as ba
    from kubernetes_cloud_amd.ops import delta_rule as dr
    from kubernetes_cloud_amd.ops import diff_attention as da
    from kubernetes_cloud_amd.ops import moe
    from kubernetes_cloud_amd.ops.norm_residual import NormedPair, prenorm
    d, _, _, sh, sg, ah, ag, dh, dg, ff, _ = SIZES[size]
    dev = torch.device("cuda", torch.cuda.current_device())
    bf = dict(device=dev, dtype=torch.bfloat16)
    i32 = dict(device=dev, dtype=torch.int32)
    R, D, out = range(ring), 128, []

    def rec(kernel, us, bytes_=0.0, flops=0.0, like=None):
        roof = max(bytes_ / HBM_TBPS / 1e6, flops / BF16_TFLOPS / 1e6)
        r = {"kernel": kernel, "us": round(us, 2), "roofline_us": round(roof, 2), "share": round(roof / us, 3), "like": like}
        out.append(r)
        print("[begopel_bench] " + json.dumps(r), file=sys.stderr, flush=True)

    # ---- norms and activation
    for n in (T, 32, 8, 1):
        xs, br, b2 = ([torch.randn(n, d, device=dev) for _ in R], *([torch.randn(n, d, **bf) for _ in R] for _ in range(2)))
        w = torch.ones(d, **bf)
        us = _time([lambda x=x, b=b: prenorm(x, b, w, 1e-5) for x, b in zip(xs, br)])
        rec(f"prenorm T={n}", us, n * d * 12, like="norm_residual")
        us = _time([lambda x=x, b=b, c=c: prenorm(x, NormedPair(b, w, c, w), w, 1e-5) for x, b, c in zip(xs, br, b2)])
        rec(f"prenorm pair T={n}", us, n * d * 14, like="norm_residual")
    u = [torch.randn(T, ff, **bf) for _ in R]
    us = _time([lambda x=x: moe.act_rows(x, x, False, act="relu2") for x in u])
    rec(f"act_rows relu2 T={T}", us, T * ff * 4, like="act_rows gated gelu")
    del u

    # ---- recurrences
    def layer(form):
        ssd = form == "ssd"
        H, G, E = (sh, sg, 64) if ssd else (dh, dg, D)
        K, V = G * STATE, H * E
        at = (0, K, 2 * K, 2 * K + 2 * V, 2 * K + V, 2 * K + 2 * V + (0 if ssd else H))  # q k v a g w
        r = lambda *s: torch.randn(*s, **bf) * 0.02  # noqa: E731
        sp = dr.DeltaHeads(False, H, G, STATE, E, at, 0, 1e-5, 4, form=form, norm_groups=G if ssd else 1)
        wt = dr.DeltaWeights(None, r(H), r(H), r(V) if ssd else r(E), conv=r(sp.conv_channels, 4),
                             conv_b=r(sp.conv_channels) if ssd else None, skip=r(H) if ssd else None)
        return sp, wt, 2 * K + 2 * V + 2 * H, V

    for form in ("head", "ssd"):
        sp, wt, cols, V = layer(form)
        for n_seq in (1, 4):
            L = T // n_seq
            ent = [(i * L, L, 0, i) for i in range(n_seq)]
            pos, slots = torch.arange(L, **i32).repeat(n_seq), torch.arange(n_seq, **i32).repeat_interleave(L)
            pl = dr.Portions(pos, slots, **{k: torch.from_numpy(v).to(dev) for k, v in dr.plan_portions(ent).items()})
            xs = [torch.randn(T, cols, **bf) for _ in R]
            st, rg = torch.zeros(n_seq, sp.state_width, device=dev), torch.zeros(n_seq, 4 * sp.conv_channels, device=dev)
            o = torch.empty(T, V, **bf)
            us = _time([lambda x=x: dr.delta_portions(sp, wt, x, st, rg, pl, o) for x in xs])
            rec(f"delta {form} T={T} in {n_seq}", us, T * (cols + V) * 2 + n_seq * sp.state_width * 4, like="delta channel")
        for B in batches:
            sts = [torch.zeros(B, sp.state_width, device=dev) for _ in range(max(2, min(8, 320 // (2 * B))))]
            rgs = [torch.zeros(B, 4 * sp.conv_channels, device=dev) for _ in sts]
            x, o = torch.randn(B, cols, **bf), torch.empty(B, V, **bf)
            pos, slots = torch.full((B,), 9, **i32), torch.arange(B, **i32)
            us = _time([lambda s=s, r=r: dr.delta_step(sp, wt, x, s, r, pos, slots, o) for s, r in zip(sts, rgs)])
            rec(f"delta_step {form} B={B}", us, B * (sp.state_width * 8 + sp.conv_channels * 16 + cols * 2 + V * 2),
                like="delta_step channel")

    # ---- biased attention
    AV, KV = ah * D, ag * D
    sp = ba.BiasedHeads(ah, ag, D, D, D ** -0.5, 1e-5, (0, AV, AV + KV, AV + 2 * KV))
    wt = ba.BiasedWeights(torch.ones(D, **bf), torch.ones(D, **bf), ba.bias_by_distance(torch.randn(BIAS[0], ah, **bf), BIAS[1]),
                          torch.zeros(ah, device=dev))
    cols = 2 * AV + 2 * KV
    for n_seq in (1, 4):
        L = T // n_seq
        pages = T // 64
        kc, vc = torch.randn(pages + 1, ag, 64, D, **bf), torch.randn(pages + 1, ag, 64, D, **bf)
        tbl = torch.arange(pages, **i32).view(n_seq, -1).contiguous()
        pos, slot = torch.arange(L, **i32).repeat(n_seq), torch.arange(n_seq, **i32).repeat_interleave(L)
        tiles = torch.from_numpy(da.plan_tiles([(i * L, L, 0, i) for i in range(n_seq)])).to(dev)
        xs, o = [torch.randn(T, cols, **bf) for _ in range(2)], torch.empty(T, AV, **bf)
        if n_seq == 1:
            us = _time([lambda x=x: ba.append(sp, wt, x, kc, vc, tbl, pos, slot) for x in xs])
            rec(f"biased_append T={T}", us, T * KV * 8, like="latent_prep")
        us = _time([lambda x=x: ba.attend_tiles(sp, wt, x, kc, vc, tbl, pos, slot, o, tiles) for x in xs])
        rec(f"biased_tile {n_seq}x{L} H={ah} G={ag}", us, 0, n_seq * (L * L / 2) * ah * 4 * D, like="latent_tile")
    for B in batches:
        nb = cached // 64
        n = max(2, min(8, int(1e9 / (B * cached * KV * 4))))
        ks, vs = ([torch.randn(B * nb + 1, ag, 64, D, **bf) for _ in range(n)] for _ in range(2))
        tbl = torch.arange(B * nb, **i32).view(B, nb).contiguous()
        pos, slot = torch.full((B,), cached - 1, **i32), torch.arange(B, **i32)
        x, o = torch.randn(B, cols, **bf), torch.empty(B, AV, **bf)
        _, _, wsf, blk = ba.rows_plan(sp, B, cached)
        ws, cnt = torch.empty(max(wsf, 1), device=dev), torch.zeros(blk, **i32)
        us = _time([lambda k=k, v=v: ba.attend_rows(sp, wt, x, k, v, tbl, pos, slot, o, cached, fused_append=True, ws=ws, cnt=cnt)
                    for k, v in zip(ks, vs)])
        rec(f"biased_rows B={B} cached={cached} H={ah} G={ag}", us, B * cached * KV * 4, like="latent decode")
        del ks, vs
    return out


def main():
    ap = argparse.ArgumentParser()
    ap.add_argument("--sizes", default="")
    ap.add_argument("--models", default="", help="gptj, rezusun, begopel")
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
