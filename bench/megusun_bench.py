#!/usr/bin/env python3
"""Megusun prefill / decode throughput beside GPT-J of equal size (the framework's closest model: parallel
residual, one norm a layer), and each kernel's distance from its roofline beside the like GPT-J kernel.

Random weights. At every size both models have the same width, vocabulary, layer count and (dense layers)
weight bytes per layer: differential attention with two maps of half GPT-J's head size over values of the full
size stores the same cache bytes a token, and a gated recurrence as wide as the model has attention's four
square projections. Through ``bench.py --megusun`` or alone:

    python bench/megusun_bench.py [--sizes ...] [--kernels]
"""
from __future__ import annotations

import argparse
import json
import os
import sys
import time

sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))

import torch

HBM_TBPS = 8.0
BF16_TFLOPS = 2500.0


def _layer(kind, d, heads, dim, mlp, kv_heads=None):
    if kind == "attention":
        mx = {"heads": heads, "kv_heads": kv_heads or heads, "dim": dim, "vdim": 2 * dim, "scale": dim ** -0.5,
              "diff": 0.4, "q_temp": {"coef": 0.1, "every": 512}}
    else:
        mx = {"width": d}
    return {"type": kind, "mixer": mx, "mlp": mlp}


def megusun_cfg(d, heads, layers, vocab, moe=None, kv_heads=None):
    """Alternating attention / recurrence; ``moe`` = (experts, top, ff, shared): the recurrence layers route."""
    dense = {"kind": "dense", "ff": 4 * d}
    routed = dense if moe is None else {"kind": "moe", "router": {"experts": moe[0], "top": moe[1]},
                                        "expert": {"ff": moe[2]}, "shared": {"ff": moe[3]}}
    dim = d // heads // 2
    return {"architecture": "Megusun", "width": d, "vocab": vocab, "norm": {"eps": 1e-5}, "residual_mult": 0.5,
            "layers": [_layer("attention", d, heads, dim, dense, kv_heads) if i % 2 == 0 else
                       _layer("mingru", d, heads, dim, routed) for i in range(layers)]}


def gptj_cfg(d, heads, layers, vocab):
    from kubernetes_cloud_amd.models.config import PRESETS_HF
    return dict(PRESETS_HF["gpt-j-6b"], n_embd=d, n_layer=layers, n_head=heads, vocab_size=vocab,
                rotary_dim=min(64, d // heads), n_positions=8192)


# name -> (width, heads, layers, vocab, experts of the routed variant, its kv heads)
SIZES = {"4096x8": (4096, 16, 8, 50400, (16, 2, 4096, 2048)), "2048x12": (2048, 16, 12, 50400, (32, 4, 1024, 1024))}


def _runs(model, vocab, prompt, batches, new_tokens, prefills):
    from kubernetes_cloud_amd.engine.llm_engine import LLMEngine, SamplingParams
    g = torch.Generator().manual_seed(0)
    out = {"prefill": [], "decode": []}
    mx = max(max(batches), max(n for n, _ in prefills))
    eng = LLMEngine(model, max_slots=mx, max_len=max(prompt + new_tokens + 80, max(t for _, t in prefills) + 1))
    for n, T in prefills:
        ids = torch.randint(0, vocab, (n, T), generator=g)
        best = 1e9
        for i in range(4):
            torch.cuda.synchronize()
            t0 = time.perf_counter()
            eng.runner.prefill(ids, list(range(n)))
            torch.cuda.synchronize()
            if i:
                best = min(best, time.perf_counter() - t0)
        for s in range(n):
            eng.runner.release(s)
        out["prefill"].append({"prompts": n, "tokens": T, "ms": round(best * 1e3, 3), "tokens_per_s": round(n * T / best)})
    for B in batches:
        prompts = [torch.randint(0, vocab, (prompt,), generator=g).tolist() for _ in range(B)]
        sp = SamplingParams(max_new_tokens=new_tokens, do_sample=False)
        eng.generate(prompts, sp)
        reqs = [eng.add_request(p, sp) for p in prompts]
        eng.step()
        torch.cuda.synchronize()
        s0, t0 = eng.stats["decode_steps"], time.perf_counter()
        eng.run_until_done(reqs)
        torch.cuda.synchronize()
        ms = (time.perf_counter() - t0) / max(1, eng.stats["decode_steps"] - s0) * 1e3
        out["decode"].append({"batch": B, "cached": prompt, "ms_per_step": round(ms, 4), "tokens_per_s": round(B / ms * 1e3),
                              "launches": eng.runner.step_launches.get(B)})
    return out


def run_models(sizes=None, batches=(1, 8, 32), prompt=1024, new_tokens=48, prefills=((1, 2048), (4, 2048)), only=None):
    from kubernetes_cloud_amd.models.causal_lm import build_model
    from kubernetes_cloud_amd.models.config import LMConfig
    dev = torch.device("cuda", torch.cuda.current_device())
    res = []
    for name in sizes or SIZES:
        d, heads, layers, vocab, moe = SIZES[name]
        for kind, cfg in (("gptj", gptj_cfg(d, heads, layers, vocab)), ("megusun", megusun_cfg(d, heads, layers, vocab)),
                          ("megusun-moe", megusun_cfg(d, heads, layers, vocab, moe, kv_heads=heads // 4))):
            if only and kind not in only:
                continue
            m = build_model(LMConfig.from_hf(cfg), device=dev, dtype=torch.bfloat16, seed=0).eval()
            r = {"size": name, "model": kind, "params_m": round(m.num_parameters() / 1e6),
                 **_runs(m, vocab, prompt, batches, new_tokens, prefills)}
            res.append(r)
            print("[megusun_bench] " + json.dumps(r), file=sys.stderr, flush=True)
            del m
            torch.cuda.empty_cache()
    return res


# ------------------------------------------------------------------------------------------- kernels
def _time(fns, reps=5):
    """us per call of a ring of calls on distinct buffers (weights and caches are cold in L2), as one HIP
    graph so that host time between launches does not count."""
    for f in fns:  # (on the stream that filled the operands)
        f()
    torch.cuda.synchronize()
    s = torch.cuda.Stream()
    with torch.cuda.stream(s):  # what the ops keep per stream
        for f in fns:
            f()
    torch.cuda.synchronize()
    g = torch.cuda.CUDAGraph()
    with torch.cuda.graph(g, stream=s):
        for f in fns:
            f()
    g.replay()
    torch.cuda.synchronize()
    best = 1e9
    for _ in range(reps):
        a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
        a.record()
        g.replay()
        b.record()
        torch.cuda.synchronize()
        best = min(best, a.elapsed_time(b))
    return best * 1e3 / len(fns)


def run_kernels(d=4096, heads=16, T=4096, cached=2048, batches=(1, 8, 32), ring=6):
    """[{kernel, us, roofline_us, share}] -- ``share`` = roofline time / measured time; ``like`` names the GPT-J
    path's kernel measured on the same sizes."""
    import torch.nn.functional as F

    from kubernetes_cloud_amd import ops
    from kubernetes_cloud_amd.ops import decode as dops
    from kubernetes_cloud_amd.ops import diff_attention as da
    from kubernetes_cloud_amd.ops import gated_scan as gs
    from kubernetes_cloud_amd.ops import moe
    from kubernetes_cloud_amd.ops.gemv import ln_rows, skinny_linear
    from kubernetes_cloud_amd.ops.rms_shift import Branch, rms_shift
    dev = torch.device("cuda", torch.cuda.current_device())
    bf = dict(device=dev, dtype=torch.bfloat16)
    i32 = dict(device=dev, dtype=torch.int32)
    out = []

    def rec(kernel, us, bytes_=0.0, flops=0.0, like=None, **kw):
        roof = max(bytes_ / HBM_TBPS / 1e6, flops / BF16_TFLOPS / 1e6)
        r = {"kernel": kernel, "us": round(us, 2), "roofline_us": round(roof, 2), "share": round(roof / us, 3), "like": like, **kw}
        out.append(r)
        print("[megusun_bench] " + json.dumps(r), file=sys.stderr, flush=True)

    R = range(ring)
    D = d // heads
    # ---- norm + shift, prompt and decode
    for n in (T, 8, 1):
        xs = [torch.randn(n, d, device=dev) for _ in R]
        br = [torch.randn(n, d, **bf) for _ in R]
        gain, mu = torch.ones((), **bf), torch.rand(d, **bf)
        one = n <= 32
        state = torch.zeros(n if one else 1, d, device=dev)
        pos = torch.arange(n, **i32) + 5
        idx = torch.arange(n, **i32) if one else torch.zeros(n, **i32)
        fl = None
        if not one:
            fl = torch.zeros(n, **i32)
            fl[0], fl[-1] = 1, 2
        prev = state if one else state.clone()
        us = _time([lambda x=x, b=b: rms_shift(x, Branch(b), .5, gain, 1e-5, shift=mu, prev=prev, prev_idx=idx, pos=pos,
                                               flags=fl, state=state, slots=idx) for x, b in zip(xs, br)])
        rec(f"rms_shift T={n}", us, n * d * (4 + 2 + 4 + 2 + 2), like="layer_norm")
        w, b2 = torch.ones(d, **bf), torch.zeros(d, **bf)
        hb, p1, p2 = ([torch.randn(n, d, **bf) for _ in R] for _ in range(3))
        if one:
            us = _time([lambda h=h, a=a, c=c: ln_rows(h, w, b2, 1e-5, (a, c)) for h, a, c in zip(hb, p1, p2)])
        else:
            us = _time([lambda h=h, a=a, c=c: ops.layer_norm(h, w, b2, 1e-5, residual=(a, c)) for h, a, c in zip(hb, p1, p2)])
        rec(f"gptj layer_norm(+2 residuals) T={n}", us, n * d * 2 * 5)
    # ---- activations and scan
    u = [torch.randn(T, 4 * d, **bf) for _ in R]
    cat = torch.empty(T, 5 * d, **bf)
    rec(f"act_rows gelu T={T}", _time([lambda x=x: moe.act_rows(x, cat[:, d:], gated=False) for x in u]), T * 4 * d * 4, like="gelu")
    rec(f"gptj gelu T={T}", _time([lambda x=x: ops.gelu(x, "tanh") for x in u]), T * 4 * d * 4)
    z = [torch.randn(T, 3 * d, **bf) for _ in R]
    bz = torch.zeros(d, **bf)
    st = torch.zeros(2, d, device=dev)
    for n_seq in (1, 4):
        ck, multi = gs.plan_chunks([(i * (T // n_seq), T // n_seq, 0, i % 2) for i in range(n_seq)])
        ck = torch.from_numpy(ck).to(dev)
        ws = torch.empty(ck.shape[0] * 3 * d, device=dev)
        us = _time([lambda x=x: gs.gated_scan(x, bz, bz, st, cat[:, :d], ck, multi, ws) for x in z])
        rec(f"gated_scan T={T} in {n_seq}", us, T * d * 8, like="gelu")
    for B in batches:
        zz = [torch.randn(B, 3 * d, **bf) for _ in R]
        ss = [torch.zeros(B, d, device=dev) for _ in R]
        p, s = torch.full((B,), 9, **i32), torch.arange(B, **i32)
        us = _time([lambda x=x, y=y: gs.gated_step(x, bz, bz, y, cat[:B, :d], p, s) for x, y in zip(zz, ss)])
        rec(f"gated_step B={B}", us, B * d * 16, like="layer_norm")
    # ---- prompt attention: one prompt of T, and four
    for G in (heads, heads // 4):
        sp = da.DiffHeads(heads, G, D // 2, D, (D // 2) ** -0.5, .5, .6, 1e-5, .1, 512.)
        for n_seq in (1, 4):
            L = T // n_seq
            pages = T // 64
            kc, vc = torch.randn(pages + 1, 2 * G, 64, D // 2, **bf), torch.randn(pages + 1, G, 64, D, **bf)
            tbl = torch.arange(pages, **i32).view(n_seq, -1).contiguous()
            pos, slot = torch.arange(L, **i32).repeat(n_seq), torch.arange(n_seq, **i32).repeat_interleave(L)
            tiles = torch.from_numpy(da.plan_tiles([(i * L, L, 0, i) for i in range(n_seq)])).to(dev)
            q = [torch.randn(T, sp.rows, **bf) for _ in range(2)]
            o = torch.empty(T, heads * D, **bf)
            us = _time([lambda x=x: da.attend_tiles(sp, x, kc, vc, tbl, pos, slot, o, tiles) for x in q])
            fl_ = n_seq * (L * L / 2) * heads * (2 * 2 * (D // 2) + 2 * 2 * D)
            rec(f"diff_tile {n_seq}x{L} H={heads} G={G}", us, 0, fl_, like="flash_attention", tflops=round(fl_ / us / 1e6))
            if G == heads:
                q5 = [torch.randn(n_seq, L, 3, heads, D, **bf) for _ in range(2)]
                us = _time([lambda x=x: ops.flash_attention(x[:, :, 0], x[:, :, 1], x[:, :, 2], causal=True) for x in q5])
                fl_ = n_seq * (L * L / 2) * heads * 4 * D
                rec(f"gptj flash_attention {n_seq}x{L} D={D}", us, 0, fl_, tflops=round(fl_ / us / 1e6))
        us = _time([lambda x=x: da.append(sp, x, kc, vc, tbl, pos, slot) for x in q])
        rec(f"diff_append T={T} G={G}", us, T * G * 2 * D * 4, like="layer_norm")
    # ---- decode attention over cold caches
    for G in (heads, heads // 4):
        sp = da.DiffHeads(heads, G, D // 2, D, (D // 2) ** -0.5, .5, .6, 1e-5, .1, 512.)
        for B in batches:  # (a grouped cache: GPT-J's kernel on the same group count)
            nb = cached // 64
            n = max(2, min(ring * 2, int(1.5e9 / (B * nb * 64 * G * 2 * D * 2))))
            ks = [torch.randn(B * nb + 1, 2 * G, 64, D // 2, **bf) for _ in range(n)]
            vs = [torch.randn(B * nb + 1, G, 64, D, **bf) for _ in range(n)]
            tbl = torch.arange(B * nb, **i32).view(B, nb).contiguous()
            pos, slot = torch.full((B,), cached - 1, **i32), torch.arange(B, **i32)
            qkv, o = torch.randn(B, sp.rows, **bf), torch.empty(B, heads * D, **bf)
            _, _, wsf, blk = da.rows_plan(sp, B, cached, torch.bfloat16)
            ws, cnt = torch.empty(max(wsf, 1), device=dev), torch.zeros(blk, **i32)
            us = _time([lambda k=k, v=v: da.attend_rows(sp, qkv, k, v, tbl, pos, slot, o, cached, fused_append=True, ws=ws,
                                                        cnt=cnt) for k, v in zip(ks, vs)])
            rec(f"diff_rows B={B} cached={cached} H={heads} G={G}", us, B * cached * G * 2 * D * 2, like="decode_attention")
            ks = [k.view(-1)[:(B * nb + 1) * G * 64 * D].view(-1, G, 64, D) for k in ks]
            q3, kl = torch.randn(B, (heads + 2 * G) * D, **bf), torch.full((B,), cached, **i32)
            w2 = torch.zeros(max(1, dops.decode_ws_floats(B, heads, G, D, cached)), device=dev)
            us = _time([lambda k=k, v=v: dops.decode_prep_attention(
                q3, heads, G, D, 0, True, None, None, pos, slot, k, v, kl, cached, out=o, ws=w2, block_table=tbl)
                for k, v in zip(ks, vs)])
            rec(f"gptj decode_attention B={B} cached={cached} G={G}", us, B * cached * G * 2 * D * 2)
            del ks, vs
    # ---- router, experts
    E, top, Fe = 16, 2, 4096
    rw, sgw = torch.randn(E, d, **bf), torch.randn(1, d, **bf)
    gu = [torch.randn(E, 2 * Fe, d, **bf) for _ in range(2)]
    dn = [torch.randn(E, d, Fe, **bf) for _ in range(2)]
    for n in (T, 32, 8, 1):
        h = torch.randn(n, d, **bf)
        mt = moe.tile_rows(n, top, E, d, Fe, torch.bfloat16)
        us = _time([lambda: moe.route_group(h, rw, top, sgw, mt) for _ in R])
        rec(f"moe_route_group T={n} E={E}", us, n * d * 2 + E * d * 2, 2. * n * d * E, like="layer_norm")
        ids, wt, _ = moe.route(h, rw, top, sgw)
        g = moe.group(ids, E, mt)
        us = _time([lambda a=a, b=b: moe.experts(h, ids, wt, a, b, g) for a, b in zip(gu, dn)])
        active = int(ids.unique().numel())
        rec(f"moe_experts T={n} E={E} top={top} F={Fe}", us, active * 3. * Fe * d * 2, 6. * n * top * Fe * d,
            like="linear", tile=mt, tflops=round(6. * n * top * Fe * d / us / 1e6))
    w = [torch.randn(4 * d, d, **bf) for _ in range(4)]
    for n in (T, 32, 8, 1):
        h = torch.randn(n, d, **bf)
        fn = (lambda x: skinny_linear(h, x)) if n == 1 else (lambda x: F.linear(h, x))
        us = _time([lambda x=x: fn(x) for x in w])
        rec(f"gptj linear T={n} N={4 * d} K={d}", us, 4. * d * d * 2, 8. * n * d * d, tflops=round(8. * n * d * d / us / 1e6))
    return out


def main():
    ap = argparse.ArgumentParser()
    ap.add_argument("--sizes", default="")
    ap.add_argument("--models", default="", help="gptj, megusun, megusun-moe")
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
