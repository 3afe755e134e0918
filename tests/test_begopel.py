"""Begopel against its plain oracle (``begopel_oracle``): every mechanism alone, then whole models through the
serving runner and engine -- prompts, decoding, portions, mixed batches, reused slots and pages, re-entered loops.

Each case runs on the CPU (the ops' reference math, which exercises cache, state and scheduler) and, marked
``gpu``, on the kernels in fp32 and bf16.
"""
import copy
import json
import math

import numpy as np
import pytest
import torch

from . import begopel_oracle as bo
from .test_rezusun import BF16, ENGINE, F32, WHERE, close, rel, rnd, runner_of, tokens, write_dir
from kubernetes_cloud_amd.engine.llm_engine import LLMEngine, SamplingParams
from kubernetes_cloud_amd.io.hf import load_pretrained, save_pretrained
from kubernetes_cloud_amd.models import begopel
from kubernetes_cloud_amd.models.causal_lm import build_model
from kubernetes_cloud_amd.models.config import LMConfig
from kubernetes_cloud_amd.ops import biased_attention as ba
from kubernetes_cloud_amd.ops import delta_rule as dr
from kubernetes_cloud_amd.ops import diff_attention as da
from kubernetes_cloud_amd.ops import moe
from kubernetes_cloud_amd.ops.norm_residual import Embedded, NormedPair, Rows, prenorm


# ------------------------------------------------------------------------------------------- configs
def ssd(heads, groups, state, vdim, conv, norm_groups=1):
    return {"type": "mamba2", "mixer": {"heads": heads, "groups": groups, "state": state, "vdim": vdim, "conv": conv,
                                        "norm_groups": norm_groups}}


def left(heads, kv_heads, dim, vdim, far, scale=None):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "bias_max": far, "scale": scale or dim ** -0.5}


def right(heads, kv_heads, dim, vdim, conv):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def both(a, b):
    return {"type": "parallel", "mixer": {"left": a, "right": b}}


def config(width, vocab, layers, eps=1e-5, scale=1.0, cap=20.0, loop=None):
    c = {"architecture": "Begopel", "width": width, "vocab": vocab, "norm": {"eps": eps}, "embedding": {"scale": scale},
         "logit_softcap": cap, "layers": [{**mx, "mlp": ff and {"kind": "dense", "ff": ff}} for mx, ff in layers]}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


CFGS = {  # name -> (config, {layer: rows of its bias table})
    # grouped heads on every side, two gated parts, a middle that runs three times, layers without a feed-forward
    "loop": (config(96, 131, [(ssd(4, 2, 24, 16, 3, 2), 120), (both(left(4, 2, 24, 40, 50, 0.31), right(4, 2, 32, 24, 4)), None),
                              (ssd(2, 1, 16, 40, 4), 88), (both(left(3, 1, 16, 16, 90), right(2, 2, 16, 32, 2)), 64)],
                    scale=1.7, loop=(1, 3, 3)), {1: 12, 3: 20}),
    # sizes no vector width divides, more parts than heads, five taps, one tap, the loop opens the model
    "odd": (config(50, 77, [(both(left(3, 3, 9, 14, 30), right(3, 1, 11, 7, 5)), 45), (ssd(3, 3, 9, 10, 1, 6), None),
                            (ssd(2, 2, 7, 13, 6, 1), 33), (both(left(2, 1, 13, 6, 24.5), right(2, 2, 10, 9, 1)), None)],
                   eps=1e-3, scale=0.25, cap=5.0, loop=(0, 2, 2)), {0: 8, 3: 6}),
    # head sizes of the matrix-core kernels, a loop to the last layer
    "wide": (config(128, 260, [(ssd(4, 2, 64, 64, 4, 4), 256), (both(left(5, 1, 80, 64, 128), right(2, 1, 80, 128, 4)), 192),
                               (both(left(4, 4, 128, 128, 200), right(4, 4, 64, 56, 3)), None), (ssd(3, 1, 128, 32, 4, 3), 64)],
                    loop=(2, 4, 2)), {1: 32, 2: 16}),
    # no loop
    "plain": (config(64, 90, [(both(left(2, 2, 32, 24, 40), right(2, 2, 24, 24, 4)), 96), (ssd(2, 1, 16, 24, 4), 64)],
                     cap=50.0), {0: 10}),
    # a loop that runs once still enters through its projection
    "once": (config(64, 90, [(ssd(2, 1, 16, 24, 4), 64), (both(left(2, 1, 32, 24, 40), right(2, 2, 24, 24, 4)), 96)],
                    scale=0.5, loop=(1, 2, 1)), {1: 10}),
}


def make(name, device, dtype, seed=0):
    cfg, rows = CFGS[name]
    w = bo.random_weights(cfg, rows, seed)
    c = begopel.with_shapes(LMConfig.from_hf(cfg), {k: tuple(v.shape) for k, v in w.items()})
    m = build_model(c, device=device, dtype=dtype, seed=None)
    m.load_state_dict({k: v.to(dtype) for k, v in begopel.to_native(w, c).items()})
    return m, w


_ORACLE = {}


def oracle(name, w, toks):
    key = (name, tuple(toks))
    if key not in _ORACLE:
        _ORACLE[key] = bo.forward(CFGS[name][0], w, toks)
    return _ORACLE[key]


# ---------------------------------------------------------------------------------------- mechanisms
@pytest.mark.parametrize("device,dtype", WHERE)
@pytest.mark.parametrize("d,T", [(64, 7), (50, 5), (1100, 3), (2052, 2), (96, 600), (700, 513), (5000, 3)])
def test_pre_norms(device, dtype, d, T):
    """Every start of a stream, every kind of branch, the rounded copy, chosen rows."""
    eps = 1e-3
    x = torch.randn(T, d, generator=torch.Generator().manual_seed(1)) * 3 + 2
    a, b = rnd(T, d, seed=2, scale=4), rnd(T, d, seed=3, scale=0.3)
    ga, gb, g, v = (rnd(d, seed=s) for s in (4, 5, 6, 7))
    dv = lambda t: t.to(device, dtype)  # noqa: E731
    tol = 2e-6 if dtype == F32 else 4e-3
    h_of = lambda s: bo.rms_about_one(s, g.double(), eps)  # noqa: E731
    plain = x.double() + a.double()
    xo, h = prenorm(x.to(device), dv(a), dv(g), eps)
    assert xo.dtype == F32 and rel(xo, plain) < 1e-6 and rel(h, h_of(plain)) < tol
    pair = x.double() + 0.5 * (bo.rms(a.double(), eps) * ga.double() + bo.rms(b.double(), eps) * gb.double())
    br = NormedPair(dv(a), dv(ga), dv(b), dv(gb))
    wide = torch.zeros(T, 2 * d + 4, device=device, dtype=dtype)
    xo, h = prenorm(x.to(device), br, dv(g), eps, raw=wide[:, 4:4 + d])
    assert rel(xo, pair) < 1e-6 and rel(h, h_of(pair)) < tol and rel(wide[:, 4:4 + d], pair) < tol
    assert float(wide[:, :4].abs().max()) == 0 and float(wide[:, 4 + d:].abs().max()) == 0
    pick = torch.tensor([T - 1, 0, T // 2], dtype=torch.int32, device=device)
    none, h = prenorm(x.to(device), br, dv(g), eps, rows=pick, keep_x=False)
    assert none is None and rel(h, h_of(pair)[[T - 1, 0, T // 2]]) < tol
    ids = torch.arange(T - 1, -1, -1, device=device)
    emb = a.double().flip(0) * 0.7
    xo, h = prenorm(Embedded(dv(a), ids, 0.7), None, dv(g), eps, raw=wide[:, :d])
    assert rel(xo, emb) < 1e-6 and rel(h, h_of(emb)) < tol and rel(wide[:, :d], emb) < tol
    start = a.double() + v.double()
    xo, h = prenorm(Rows(dv(torch.cat([a, a], 1))[:, :d], dv(v)), dv(b), dv(g), eps)
    assert rel(xo, start + b.double()) < 1e-6 and rel(h, h_of(start + b.double())) < tol
    xo, none = prenorm(x.to(device), dv(a), None, eps)
    assert none is None and rel(xo, plain) < 1e-6


@pytest.mark.parametrize("device,dtype", WHERE)
@pytest.mark.parametrize("F", [48, 37])
def test_squared_relu_and_softcap(device, dtype, F):
    x = rnd(6, F, seed=50, scale=3)
    y = torch.empty(6, F, device=device, dtype=dtype)
    tol = 1e-6 if dtype == F32 else 4e-3
    assert rel(moe.act_rows(x.to(device, dtype), y, False, act="relu2"), torch.relu(x.double()) ** 2) < tol
    z = x.to(device, dtype) * 4
    assert rel(moe.act_rows(z, z, False, act="softcap", cap=7.0), bo.softcap(4 * x.double(), 7.0)) < tol


@pytest.mark.gpu
@pytest.mark.parametrize("rows", [1, 2, 7, 16, 40])
def test_squared_relu_behind_a_product(rows):
    """In the streaming products' epilogues and behind the library product."""
    m, _ = make("wide", "cuda", BF16)
    r = runner_of(m, max_slots=1, max_len=64)
    x, w = rnd(rows, 128, seed=1), rnd(256, 128, seed=2, scale=0.1)
    got = r._linear(x.cuda().to(BF16), w.cuda().to(BF16), act=3)
    assert rel(got, torch.relu(x.double() @ w.double().T) ** 2) < 6e-3


@pytest.mark.parametrize("rows,far", [(32, 128), (16, 256), (8, 64), (24, 1000), (12, 27), (6, 24.5), (2, 9)])
def test_distance_buckets(rows, far):
    """The product's buckets, its table by distance and the oracle's agree, with exact edges by integers."""
    half = rows // 2
    table = torch.arange(rows).float()[:, None].expand(rows, 3).contiguous()
    flat = ba.bias_by_distance(table, far)
    for n in range(int(far) + 20):
        b = ba.distance_bucket(n, rows, far)
        assert b == bo.distance_bucket(n, rows, far) == float(flat[1, min(n, flat.shape[1] - 1)])
        if n >= half and isinstance(far, int):  # b - half = floor(m ln(n / half) / ln(far / half)), m = rows - half
            m = rows - half
            ge = lambda k: n ** m * half ** k >= far ** k * half ** m  # noqa: E731
            assert ge(b - half) and (b == rows - 1 or not ge(b - half + 1))
    assert ba.distance_bucket(half - 1, rows, far) == half - 1 and float(flat[0, -1]) == rows - 1


class Biased:
    """One attention layer on given projection rows, through the paged ops."""

    def __init__(self, m, rows, T, seed=0):
        H, G, D, E = (m[k] for k in ("heads", "kv_heads", "dim", "vdim"))
        names = {"q": H * D, "k": G * D, "v": G * E, "g": H * E}
        at, o = {}, 0
        for n, c in names.items():
            at[n] = o
            o += -(-c // 8) * 8
        self.m, self.at, self.names = m, at, names
        self.x = rnd(T, o, seed=seed + 1)
        w = {"q.norm": 1 + 0.3 * rnd(D, seed=seed + 2), "k.norm": 1 + 0.3 * rnd(D, seed=seed + 3), "rel": 1.5 * rnd(rows, H, seed=seed + 4),
             "sink": 1 + rnd(H, seed=seed + 5)}
        self.w = {k: v.to(BF16).double() for k, v in w.items()}
        for n, c in names.items():
            self.w[n] = torch.zeros(c, o).double()
            self.w[n][torch.arange(c), at[n] + torch.arange(c)] = 1
        self.w["o"] = torch.eye(H * E).double()
        self.sp = ba.BiasedHeads(H, G, D, E, m["scale"], 1e-5, tuple(at[n] for n in "qkvg"))

    def cols(self, n):
        return self.x[:, self.at[n]:self.at[n] + self.names[n]]

    def want(self, x):
        return bo.biased_attention(x.double(), self.w, "", self.m, 1e-5)

    def weights(self, device, dtype):
        w = self.w
        return ba.BiasedWeights(w["q.norm"].to(device, dtype), w["k.norm"].to(device, dtype),
                                ba.bias_by_distance(w["rel"].to(device), self.m["bias_max"]), w["sink"].float().to(device))

    def run(self, cuts, device, dtype, PS=64, beside=None):
        """The first sequence by portions ``cuts``; ``beside`` shares its batches."""
        sp, T, wt = self.sp, self.x.shape[0], self.weights(device, dtype)
        nb = -(-T // PS) + 1
        kp = torch.full((2 * nb + 1, sp.kv_heads, PS, sp.dim), 50.0, device=device, dtype=dtype)
        vp = torch.full((2 * nb + 1, sp.kv_heads, PS, sp.vdim), 50.0, device=device, dtype=dtype)
        perm = torch.randperm(2 * nb, generator=torch.Generator().manual_seed(3)).int()
        table = torch.cat([perm.view(2, nb), torch.full((1, nb), 2 * nb).int()]).to(device)
        outs, at = [], 0
        for n in cuts:
            rows, ent = [self.x[at:at + n]], [(0, n, at, 1)]
            if beside is not None and at + n <= beside.shape[0]:
                rows.append(beside[at:at + n])
                ent.append((n, n, at, 0))
            x = torch.cat(rows).to(device, dtype)
            i32 = lambda v: torch.as_tensor(np.asarray(v), dtype=torch.int32).to(device)  # noqa: E731
            pos = i32(np.concatenate([np.arange(p, p + c) for _, c, p, _ in ent]))
            slot = i32(np.repeat([e[3] for e in ent], [e[1] for e in ent]))
            out = torch.zeros(x.shape[0], sp.heads * sp.vdim + 16, device=device, dtype=dtype)
            a = (sp, wt, x, kp, vp, table, pos, slot, out[:, :-16])
            if n == 1:
                ba.attend_rows(*a, at + 1, fused_append=True)
            else:
                ba.append(*a[:-1])
                if device == "cuda" and ba.tiles_ok(sp, dtype, PS, x.stride(0), out.stride(0)):
                    ba.attend_tiles(*a, i32(da.plan_tiles(ent)))
                else:
                    ba.attend_rows(*a, at + n, fused_append=False)
            assert float(out[:, -16:].abs().max()) == 0
            outs.append(out[:n, :-16])
            at += n
        assert at == T
        return torch.cat(outs)


BIASED = {"grouped": (left(6, 2, 32, 48, 60), 16), "odd": (left(3, 1, 9, 14, 30), 6), "one": (left(1, 1, 16, 16, 20, 0.4), 8),
          "many": (left(10, 1, 24, 16, 100, 0.5), 12), "big": (left(2, 2, 128, 256, 77), 32), "tall": (left(4, 2, 96, 64, 500), 10),
          "flat": (left(2, 1, 40, 136, 12), 2)}


@pytest.mark.parametrize("device,dtype", WHERE)
@pytest.mark.parametrize("kind", list(BIASED))
def test_biased_attention(device, dtype, kind):
    d = Biased(*BIASED[kind], 140)
    other = rnd(60, d.x.shape[1], seed=12)
    want = d.want(d.x)
    tol = 5e-6 if dtype == F32 else 2e-2
    for cuts, PS in (([140], 64), ([2, 63, 2, 1, 1, 33, 38], 64), ([31, 1, 32, 64, 1, 11], 16), ([100] + [1] * 40, 32)):
        got = d.run(cuts, device, dtype, PS, beside=other)
        assert rel(got, want) < tol, (cuts, rel(got, want))
        assert rel(got[:2], want[:2]) < tol


@pytest.mark.gpu
@pytest.mark.parametrize("dim", [8, 40, 64, 96, 128])
@pytest.mark.parametrize("vdim", [24, 64, 88, 128, 200])
def test_biased_tile_sizes(dim, vdim):
    """Every matrix-core instance, a portion in mid-page, bias rows short, long, and too long to be staged."""
    for far, rows in ((20, 8), (700, 64), (200000, 6)):
        d = Biased(left(2, 1, dim, vdim, far), rows, 150, seed=90)
        assert ba.tiles_ok(d.sp, BF16, 64, d.x.shape[1], 2 * vdim + 16)
        want = d.want(d.x)
        assert rel(d.run([150], "cuda", BF16), want) < 2e-2
        assert rel(d.run([37, 113], "cuda", BF16), want) < 2e-2


@pytest.mark.parametrize("device,dtype", WHERE)
@pytest.mark.parametrize("row", [0, 1, 5, 7, 8, 9, 12, 15])
def test_one_bucket_stands_out(device, dtype, row):
    """A single row of the bias table takes the whole weight: keys just inside and just outside each of its edges
    (one distance, a range, everything beyond) change the output completely."""
    d = Biased(left(2, 1, 32, 32, 90), 16, 200, seed=30)
    d.w["rel"][:] = 0
    d.w["rel"][row] = torch.tensor([9.0, -9.0]).double()
    want = d.want(d.x)
    tol = 1e-5 if dtype == F32 else 2.5e-2
    for cuts in ([200], [64, 64, 2, 70], [190] + [1] * 10):
        got = d.run(cuts, device, dtype)
        for h in range(2):
            s = slice(32 * h, 32 * h + 32)
            assert rel(got[:, s], want[:, s]) < tol and rel(got[-10:, s], want[-10:, s]) < tol, (cuts, h)


@pytest.mark.parametrize("device,dtype", WHERE)
@pytest.mark.parametrize("key", [0, 1, 63, 64, 65, 127, 128, 200, 254])
def test_one_key_stands_out(device, dtype, key):
    """A far key takes a head's whole weight; the last token holds a larger one that only it may see."""
    d = Biased(left(2, 1, 32, 32, 60, 1.0), 16, 257, seed=40)
    d.w["q.norm"].fill_(1)
    d.w["k.norm"].fill_(1)
    q, k = d.cols("q"), d.cols("k")
    q[255:] = 0
    q[255:, 3] = q[255:, 35] = 5.0
    k[:, 3] = 0
    k[key], k[256] = 0, 0
    k[key, 3] = 3.0
    k[256, 3] = 4.0
    k[256, 4] = 0.5
    want = d.want(d.x)
    tol = 1e-5 if dtype == F32 else 2.5e-2
    for cuts in ([257], [255, 2], [255, 1, 1], [128, 127, 2], [64, 64, 64, 63, 1, 1]):
        got = d.run(cuts, device, dtype)
        assert rel(got[255:], want[255:]) < tol and rel(got[:255], want[:255]) < tol, cuts


@pytest.mark.parametrize("device,dtype", WHERE)
def test_sink_and_gate(device, dtype):
    """A large sink empties a head, a very negative one leaves a plain softmax -- from the first token on; a closed
    gate closes its columns only."""
    d = Biased(left(3, 3, 32, 32, 60), 8, 80, seed=50)
    d.w["sink"][:] = torch.tensor([12.0, -30.0, 0.0]).double()
    d.cols("g")[:, 40:50] = -20
    want = d.want(d.x)
    assert float(want[0, :32].abs().max()) < 0.2 * float(want[0, 50:64].abs().max())
    for cuts in ([80], [2, 78], [1] * 8 + [72]):
        got = d.run(cuts, device, dtype)
        assert float(got[:, 40:50].abs().max()) < 1e-6
        for h in range(3):
            s = slice(32 * h, 32 * h + 32)
            assert rel(got[:, s], want[:, s]) < (1e-5 if dtype == F32 else 2.5e-2), (cuts, h)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("shape", [(8, 2, 64, 64), (9, 3, 96, 80), (3, 3, 24, 40), (5, 1, 11, 13), (2, 1, 128, 256)])
def test_biased_decode_over_key_splits(dtype, shape):
    """Rows of unequal length over a long cache cut in splits."""
    H, G, D, E = shape
    d = Biased(left(H, G, D, E, 300), 32, 4, seed=70)
    sp, wt = d.sp, d.weights("cuda", dtype)
    lens, PS = [1500, 1, 257, 513], 64
    g = torch.Generator().manual_seed(5)
    nb = [-(-n // PS) for n in lens]
    kp, vp = (torch.full((sum(nb) + 1, G, PS, n), 40.0).to(BF16) for n in (D, E))
    table = torch.full((5, max(nb)), sum(nb), dtype=torch.int32)
    at, ks, vs = 0, [], []
    for b, n in enumerate(lens):
        table[b, :nb[b]] = torch.arange(at, at + nb[b])
        k, v = torch.randn(n, G, D, generator=g).to(BF16), torch.randn(n, G, E, generator=g).to(BF16)
        for i in range(nb[b]):
            kk, vv = k[i * PS:(i + 1) * PS], v[i * PS:(i + 1) * PS]
            kp[at + i, :, :kk.shape[0]], vp[at + i, :, :vv.shape[0]] = kk.transpose(0, 1), vv.transpose(0, 1)
        at += nb[b]
        ks.append(k.double())
        vs.append(v.double())
    want = torch.empty(4, H, E).double()
    for b, n in enumerate(lens):
        x = d.x[b].double()
        part = lambda name, c: x[d.at[name]:d.at[name] + d.names[name]].view(-1, c)  # noqa: E731
        q = bo.rms(part("q", D), 1e-5) * d.w["q.norm"]
        ks[b][-1] = bo.rms(part("k", D), 1e-5) * d.w["k.norm"]
        vs[b][-1] = part("v", E)
        bias = torch.stack([d.w["rel"][bo.distance_bucket(i, 32, 300)] for i in range(n)]).flip(0)
        for h in range(H):
            s = ks[b][:, h * G // H] @ q[h] * sp.scale + bias[:, h]
            want[b, h] = bo.sink_softmax_row(s, d.w["sink"][h]) @ vs[b][:, h * G // H]
        want[b] *= torch.sigmoid(part("g", E))
    assert ba.rows_plan(sp, 4, 1500)[0] > 1
    pos = torch.tensor([n - 1 for n in lens], dtype=torch.int32).cuda()
    out = torch.zeros(4, H * E, device="cuda", dtype=dtype)
    a = (sp, wt, d.x.to("cuda", dtype), kp.to("cuda", dtype), vp.to("cuda", dtype), table.cuda(), pos,
         torch.arange(4, dtype=torch.int32).cuda())
    for _ in range(2):
        ba.attend_rows(*a, out, 1500, fused_append=True)
        assert rel(out, want.view(4, -1)) < (1e-5 if dtype == F32 else 2e-2)
    one = torch.zeros_like(out)
    ba.attend_rows(*a, one, 1500, fused_append=False, row_of=torch.tensor([2], dtype=torch.int32, device="cuda"))
    assert rel(one[2], want.view(4, -1)[2]) < (1e-5 if dtype == F32 else 2e-2) and float(one[[0, 1, 3]].abs().max()) == 0


class Recurrence:
    """One gated delta rule or state-space layer on given projection rows, and the oracle with identity projections
    over the same rows."""

    def __init__(self, kind, m, T, seed=0, tweak=None):
        self.ssd, self.m = kind == "ssd", m
        H, E, taps = m["heads"], m["vdim"], m["conv"]
        if self.ssd:
            G, D = m["groups"], m["state"]
            names, order = {"C": G * D, "B": G * D, "x": H * E, "z": H * E, "dt": H}, ("C", "B", "x", "dt", "z", "dt")
        else:
            G, D = m["kv_heads"], m["dim"]
            names, order = {"q": G * D, "k": G * D, "v": H * E, "g": H * E, "b": H, "a": H}, ("q", "k", "v", "b", "g", "a")
        at, o = {}, 0
        for n, c in names.items():
            at[n] = o
            o += -(-c // 8) * 8
        self.names, self.at = names, at
        self.x = rnd(T, o, seed=seed + 1)
        self.sp = dr.DeltaHeads(False, H, G, D, E, tuple(at[n] for n in order), 0, 1e-5, taps, form="ssd" if self.ssd else "head",
                                norm_groups=m.get("norm_groups", 1))
        pick = lambda n: torch.nn.functional.one_hot(torch.arange(at[n], at[n] + names[n]), o).double()  # noqa: E731
        w = {"A_log": rnd(H, seed=seed + 2, scale=0.7) - 0.5, "dt_bias": rnd(H, seed=seed + 3, scale=1.5) - 2,
             "norm": 1 + 0.3 * rnd(H * E if self.ssd else E, seed=seed + 4)}
        if self.ssd:
            n = H * E + 2 * G * D
            w.update({"conv": rnd(n, taps, seed=seed + 5, scale=0.7), "conv.b": rnd(n, seed=seed + 6, scale=0.7), "D": rnd(H, seed=seed + 7)})
        else:
            w.update({c + ".conv": rnd(names[c], taps, seed=seed + 5 + i, scale=0.7) for i, c in enumerate("qkv")})
        self.w = {k: v.to(BF16).double() for k, v in w.items()}
        if tweak:
            tweak(self)
        if self.ssd:
            self.w["in"] = torch.cat([pick(n) for n in ("z", "x", "B", "C", "dt")])
        else:
            self.w.update({n: pick(n) for n in names})
        self.w["o"] = torch.eye(H * E).double()

    def cols(self, n):
        return self.x[:, self.at[n]:self.at[n] + self.names[n]]

    def want(self, x):
        return (bo.ssd if self.ssd else bo.head_delta)(x.double(), self.w, "", self.m, 1e-5)

    def weights(self, dv):
        w = self.w
        if not self.ssd:
            return dr.DeltaWeights(None, dv(w["dt_bias"]), dv(w["A_log"]), dv(w["norm"]),
                                   conv=dv(torch.cat([w[n + ".conv"] for n in "qkv"])))
        n, s = self.names["x"], self.names["B"]
        turn = lambda t: torch.cat([t[n + s:], t[n:n + s], t[:n]])  # noqa: E731  (x, B, C -> C, B, x)
        return dr.DeltaWeights(None, dv(w["dt_bias"]), dv(w["A_log"]), dv(w["norm"]), conv=dv(turn(w["conv"])),
                               conv_b=dv(turn(w["conv.b"])), skip=dv(w["D"]))

    def state(self, slots, device):
        sp = self.sp
        return (torch.full((slots, sp.state_width), 7.0, device=device),
                torch.full((slots, sp.taps * sp.conv_channels), -5.0, device=device))

    def run(self, batch, wt, S, ring, device, dtype):
        """One batch of [(rows [n, cols], position, slot)] -> outputs [sum n, H dv]."""
        x = torch.cat([b[0] for b in batch]).to(device, dtype)
        ent, r = [], 0
        for rows, pos, slot in batch:
            ent.append((r, rows.shape[0], pos, slot))
            r += rows.shape[0]
        i32 = lambda v: torch.as_tensor(np.asarray(v), dtype=torch.int32).to(device)  # noqa: E731
        pos = i32(np.concatenate([np.arange(p, p + n) for _, n, p, _ in ent]))
        slots = i32(np.repeat([e[3] for e in ent], [e[1] for e in ent]))
        out = torch.zeros(r, self.sp.heads * self.sp.vdim + 8, device=device, dtype=dtype)
        y = out[:, :-8]
        if all(e[1] == 1 for e in ent):
            dr.delta_step(self.sp, wt, x, S, ring, pos, slots, y)
        else:
            pl = dr.Portions(pos, slots, **{k: i32(v) for k, v in dr.plan_portions(ent).items()})
            dr.delta_portions(self.sp, wt, x, S, ring, pl, y)
        assert float(out[:, -8:].abs().max()) == 0
        return y


RECURRENCES = {
    "head": ("head", right(4, 2, 32, 48, 4)), "head-odd": ("head", right(3, 1, 9, 14, 5)), "head-128": ("head", right(2, 2, 128, 128, 4)),
    "head-tall": ("head", right(2, 1, 128, 24, 3)), "head-flat": ("head", right(2, 2, 40, 128, 1)), "head-taps": ("head", right(2, 2, 32, 32, 6)),
    "head-200": ("head", right(1, 1, 200, 64, 4)),
    "ssd": ("ssd", ssd(4, 2, 32, 48, 4, 2)["mixer"]), "ssd-odd": ("ssd", ssd(3, 3, 9, 14, 5, 6)["mixer"]),
    "ssd-128": ("ssd", ssd(4, 1, 128, 64, 4, 4)["mixer"]), "ssd-wide": ("ssd", ssd(2, 1, 16, 128, 2, 1)["mixer"]),
    "ssd-taps": ("ssd", ssd(6, 3, 48, 16, 6, 3)["mixer"]), "ssd-one": ("ssd", ssd(8, 2, 64, 24, 1, 16)["mixer"]),
    "ssd-256": ("ssd", ssd(2, 2, 256, 32, 4, 1)["mixer"])}


@pytest.mark.parametrize("device,dtype", WHERE)
@pytest.mark.parametrize("kind", list(RECURRENCES))
def test_recurrences(device, dtype, kind):
    """Portions (one token to several chunks, cut anywhere) of two sequences continue one recurrence; the slots
    held something else before."""
    lens = [190, 61]
    d = Recurrence(*RECURRENCES[kind], sum(lens))
    wt = d.weights(lambda t: t.to(device, dtype))
    seqs = d.x.split(lens)
    want = [d.want(s) for s in seqs]
    tol = 1e-5 if dtype == F32 else 2e-2
    plans = [[[(0, 190), (1, 61)]], [[(0, 64), (1, 2)], [(1, 3), (0, 65)], [(0, 2)], [(0, 1), (1, 1)], [(0, 15), (1, 55)], [(0, 43)]],
             [[(0, 63), (1, 17)], [(0, 1), (1, 1)], [(0, 1), (1, 1)], [(0, 124), (1, 1)], [(0, 1), (1, 41)]],
             [[(0, 130)], [(1, 33), (0, 60)], [(1, 28)]]]
    for plan in plans:
        S, ring = d.state(4, device)
        at, got = [0, 0], [[], []]
        for batch in plan:
            y = d.run([(seqs[s][at[s]:at[s] + n], at[s], 2 - s) for s, n in batch], wt, S, ring, device, dtype)
            for (s, n), o in zip(batch, y.split([n for _, n in batch])):
                got[s].append(o)
                at[s] += n
        for s in (0, 1):
            g = torch.cat(got[s])
            assert g.shape[0] == lens[s] and rel(g, want[s]) < tol, (plan, s, rel(g, want[s]))
            assert rel(g[-2:], want[s][-2:]) < tol and rel(g[:4], want[s][:4]) < tol
        assert float(S[3].sub(7).abs().max()) == 0 and float(S[0].sub(7).abs().max()) == 0  # other slots untouched


@pytest.mark.gpu
@pytest.mark.parametrize("state,vdim,heads", [(40, 32, 130), (104, 32, 128), (48, 64, 192), (128, 56, 200)])
def test_many_state_space_heads(state, vdim, heads):
    """Enough heads that a workgroup takes several column tiles."""
    d = Recurrence("ssd", ssd(heads, 2, state, vdim, 4, 2)["mixer"], 80, seed=80)
    wt = d.weights(lambda t: t.to("cuda", BF16))
    S, ring = d.state(3, "cuda")
    got = d.run([(d.x, 0, 1), (d.x[:70], 0, 2)], wt, S, ring, "cuda", BF16)
    want = d.want(d.x)
    assert rel(got[:80], want) < 2e-2 and rel(got[80:], want[:70]) < 2e-2
    got = d.run([(d.x[70:], 70, 2)], wt, S, ring, "cuda", BF16)
    assert rel(got, want[70:]) < 2e-2


@pytest.mark.parametrize("device,dtype", WHERE)
@pytest.mark.parametrize("kind", ["head", "head-128", "ssd", "ssd-128"])
def test_long_recurrent_decoding(device, dtype, kind):
    d = Recurrence(*RECURRENCES[kind], 150, seed=20)
    wt = d.weights(lambda t: t.to(device, dtype))
    S, ring = d.state(2, device)
    got = torch.cat([d.run([(d.x[t:t + 1], t, 1)], wt, S, ring, device, dtype) for t in range(150)])
    assert rel(got, d.want(d.x)) < (1e-5 if dtype == F32 else 1.2e-2)


@pytest.mark.parametrize("device,dtype", WHERE)
@pytest.mark.parametrize("kind", ["head", "ssd"])
@pytest.mark.parametrize("at", [0, 1, 15, 16, 63, 64, 100, 127, 128])
def test_one_write_stands_out(device, dtype, kind, at):
    """Nearly no decay, one token writes a large value and the tokens after 130 read its key: a write that gets
    lost at a chunk's or portion's edge, or is seen by the token before it, changes the output."""
    q, k, v = ("C", "B", "x") if kind == "ssd" else ("q", "k", "v")

    def still(d):
        d.w["dt_bias"].fill_(-4)
        d.w["A_log"].fill_(-6)
        for n in ("dt",) if d.ssd else ("a",):
            d.cols(n)[:] = 0
        for n in ("conv", "conv.b") if d.ssd else [c + ".conv" for c in "qkv"]:
            d.w[n].zero_()
            if not n.endswith(".b"):
                d.w[n][:, -1] = 1
        if d.ssd:
            d.w["D"].zero_()
        for n in (k, v):
            d.cols(n)[:] *= 0.02
        D, E = d.sp.dim, d.sp.vdim
        key = rnd(D, seed=77).abs() + 0.5
        d.cols(q)[130:, :D] = key
        d.cols(k)[at, :D] = key
        d.cols(v)[at, :E] = rnd(E, seed=78, scale=4)
        d.cols(q)[at - 1 if at else 1, :D] = key
        if not d.ssd:
            d.cols("b")[:] = -6  # the others write weakly
            d.cols("b")[at] = 6

    d = Recurrence(*RECURRENCES[kind], 140, seed=40, tweak=still)
    wt = d.weights(lambda t: t.to(device, dtype))
    want = d.want(d.x)
    tol = 2e-5 if dtype == F32 else 2.5e-2
    for cuts in ([140], [64, 64, 12], [at + 1, 139 - at], [128, 2, 10], [100] + [1] * 40):
        S, ring = d.state(2, device)
        got, t = [], 0
        for n in cuts:
            if n:
                got.append(d.run([(d.x[t:t + n], t, 0)], wt, S, ring, device, dtype))
                t += n
        got = torch.cat(got)
        assert rel(got[130:], want[130:]) < tol and rel(got, want) < 2 * tol, cuts
        near = slice(max(0, at - 1), at + 1)
        assert rel(got[near], want[near]) < 3 * tol, cuts


@pytest.mark.parametrize("device,dtype", WHERE)
@pytest.mark.parametrize("kind", ["head-128", "ssd-128"])
def test_fast_and_slow_decays(device, dtype, kind):
    """A head that forgets within a token beside one that never does."""
    def fast(d):
        d.w["dt_bias"][::2] = 30.0
        d.w["dt_bias"][1::2] = -8.0
        d.w["A_log"].fill_(2.0)

    d = Recurrence(*RECURRENCES[kind], 200, seed=60, tweak=fast)
    wt = d.weights(lambda t: t.to(device, dtype))
    S, ring = d.state(2, device)
    got = d.run([(d.x, 0, 1)], wt, S, ring, device, dtype)
    assert rel(got, d.want(d.x)) < (1e-5 if dtype == F32 else 2e-2)


# -------------------------------------------------------------------------------------------- models
@pytest.mark.parametrize("device,dtype", WHERE)
@pytest.mark.parametrize("name", list(CFGS))
def test_prompt_decode_and_portions(device, dtype, name):
    """The same logits for a whole prompt, token by token, and cut in portions down to two tokens."""
    m, w = make(name, device, dtype)
    toks = tokens(140, CFGS[name][0]["vocab"], 1)
    want = oracle(name, w, toks)
    r = runner_of(m, max_slots=2, max_len=192)
    for cuts in ([140], [1] * 70 + [70], [2, 3, 61, 2, 31, 1, 40], [129, 1, 1, 1, 8]):
        at, got = 0, []
        for n in cuts:
            got.append(r.forward_tokens([(1, toks[at:at + n], at, range(n))]))
            at += n
        close(torch.cat(got), want, dtype)
        r.release(1)


@pytest.mark.parametrize("device,dtype", WHERE)
@pytest.mark.parametrize("name", list(CFGS))
def test_residual_stream_after_every_run(device, dtype, name):
    """The stream after every layer run, a looped layer counted each time."""
    m, w = make(name, device, dtype)
    toks = tokens(40, CFGS[name][0]["vocab"], 2)
    got, want = [], []
    runner_of(m, max_slots=1, max_len=64).forward_tokens([(0, toks, 0, [39])], got)
    bo.forward(CFGS[name][0], w, toks, want)
    assert len(got) == len(want) == len(m.cfg.runs)
    for i, (a, b) in enumerate(zip(got, want)):
        assert a.dtype == F32  # the residual sum
        assert rel(a, b) < (3e-6 if dtype == F32 else 0.04), i


def test_passes_have_their_own_cache_and_state():
    m, _ = make("loop", "cpu", F32)
    r = runner_of(m, max_slots=1, max_len=64)
    assert m.cfg.runs == (0, 1, 2, 1, 2, 1, 2, 3) and m.cfg.opens == (None, 0, None, 1, None, 2, None, None)
    assert len(r.cache.k) == 4 and len(r.state.t) == 2 * 8
    lefts = [r.mixers[i].sides[0] for i in (1, 3, 5)]
    assert lefts[0].wt is lefts[1].wt and len({x.index for x in lefts}) == 3
    assert make("once", "cpu", F32)[0].cfg.opens == (None, 0) and make("plain", "cpu", F32)[0].cfg.opens == (None, None)
    assert make("odd", "cpu", F32)[0].cfg.opens == (0, None, 1, None, None, None)
    for bad in ((1, 9, 2), (3, 2, 1)):
        c = copy.deepcopy(CFGS["odd"][0])
        c["loop"] = dict(zip(("start", "stop", "times"), bad))
        with pytest.raises(ValueError, match="loop"):
            LMConfig.from_hf(c)


@pytest.mark.parametrize("device,dtype", WHERE)
@pytest.mark.parametrize("name", ["loop", "wide"])
def test_mixed_batches_and_reused_slots(device, dtype, name):
    """Unequal requests share batches (portions beside single tokens), slots and pages turn over in a pool too
    small for all of them, and each request's logits are those it has alone."""
    m, w = make(name, device, dtype)
    PS = 16 if name == "loop" else 32
    r = runner_of(m, max_slots=3, max_len=128, page_size=PS, kv_pages=224 // PS)
    lens = {"a": 100, "b": 70, "c": 3, "d": 1, "e": 95, "f": 40}
    if name == "wide":
        lens = {"a": 90, "b": 64, "c": 2, "d": 50}
    seqs = {i: tokens(n, CFGS[name][0]["vocab"], 60 + k) for k, (i, n) in enumerate(lens.items())}
    want = {i: oracle(name, w, t) for i, t in seqs.items()}
    g = torch.Generator().manual_seed(9)
    waiting, live, free, got = list(seqs), {}, [0, 1, 2], {i: [] for i in seqs}
    while waiting or live:
        while waiting and free:
            if live and torch.rand(1, generator=g) < 0.3:
                break
            live[waiting.pop(0)] = [free.pop(), 0]
        batch, names = [], []
        for i, (slot, at) in live.items():
            if len(live) > 1 and torch.rand(1, generator=g) < 0.2 and batch:
                continue  # left out of this step
            n = int([1, 1, 2, 5, 17, 33][int(torch.randint(0, 6, (1,), generator=g))])
            n = min(n, lens[i] - at)
            batch.append((slot, seqs[i][at:at + n], at, range(n)))
            names.append((i, n))
        out = r.forward_tokens(batch).split([n for _, n in names])
        for (i, n), o in zip(names, out):
            got[i].append(o)
            live[i][1] += n
            if live[i][1] == lens[i]:
                slot = live.pop(i)[0]
                r.release(slot)
                free.append(slot)
    for i in seqs:
        close(torch.cat(got[i]), want[i], dtype)
    assert r.cache.free_count() == 224 // PS


@pytest.mark.parametrize("device,dtype", WHERE)
@pytest.mark.parametrize("name", ["wide", "odd"])
def test_long_decoding(device, dtype, name):
    """Token by token across several pages, after a one-token prompt."""
    m, w = make(name, device, dtype)
    n = 90 if device == "cpu" else 230
    toks = tokens(n, CFGS[name][0]["vocab"], 4)
    r = runner_of(m, max_slots=1, max_len=256)
    got = torch.cat([r.forward_tokens([(0, [t], i, [0])]) for i, t in enumerate(toks)])
    close(got, oracle(name, w, toks), dtype)


@pytest.mark.parametrize("device,dtype", WHERE)
def test_first_tokens_do_not_see_the_slot_before(device, dtype):
    """A sequence in a slot (and pages) just used by another starts from nothing: no state, no convolution input."""
    m, _ = make("wide", device, dtype)
    r = runner_of(m, max_slots=1, max_len=64, kv_pages=1)
    toks = tokens(20, 260, 5)
    first = r.forward_tokens([(0, toks, 0, range(20))])
    r.release(0)
    r.forward_tokens([(0, tokens(60, 260, 6), 0, [])])
    r.release(0)
    assert torch.equal(first, r.forward_tokens([(0, toks, 0, range(20))]))
    one = torch.cat([r.forward_tokens([(0, [t], i, [0])]) for i, t in enumerate(toks[:6])])
    close(one, first[:6].double().cpu(), dtype)


def greedy(name, w, prompt, n):
    ids = list(prompt)
    for _ in range(n):
        ids.append(int(bo.forward(CFGS[name][0], w, ids)[-1].argmax()))
    return ids[len(prompt):]


@pytest.mark.parametrize("device,graphs", ENGINE)
def test_engine_greedy(device, graphs):
    """Greedy generation through the engine: whole prompts, chunked prompts in mixed steps, more requests than
    slots, the lookahead decode (and its HIP graphs) -- the oracle's tokens each time."""
    name = "loop"
    m, w = make(name, device, F32)
    prompts = [tokens(n, CFGS[name][0]["vocab"], 70 + n) for n in (5, 33, 1, 12, 21)]
    want = [greedy(name, w, p, 6) for p in prompts]
    sp = SamplingParams(max_new_tokens=6, do_sample=False)
    for kw in ({}, {"prefill_chunk": 7}, {"prefill_chunk": 2, "max_slots": 2}, {"pipeline": False}):
        eng = LLMEngine(m, max_len=64, use_graphs=graphs, **{"max_slots": 5, **kw})
        reqs = [eng.add_request(prompts[0], sp)]
        eng.step()  # one request runs before the others arrive
        reqs += [eng.add_request(p, sp) for p in prompts[1:]]
        eng.run_until_done(reqs)
        assert [r.output for r in reqs] == want, kw
        assert bool(eng.stats["mixed_steps"]) == ("prefill_chunk" in kw)
        assert len(eng.free) == eng.runner.max_slots and eng.runner.cache.free_count() == eng.runner.cache.n_pages
        again = eng.generate(prompts, sp)  # warm graphs, used slots
        assert [r.output for r in again] == want, kw


@pytest.mark.gpu
def test_graph_steps_match_eager_in_bf16():
    """Replayed decode graphs advance state and cache exactly as eager steps do, batch sizes changing from step to
    step."""
    m, _ = make("wide", "cuda", BF16)
    sp = [SamplingParams(max_new_tokens=n, do_sample=True, temperature=0.9, top_k=20, seed=s, repetition_penalty=1.2,
                         logprobs=True) for n, s in ((12, 1), (5, 2), (20, 3), (9, 4))]
    prompts = [tokens(n, 260, n) for n in (4, 40, 17, 70)]
    outs = []
    for graphs in (False, True, True):
        eng = LLMEngine(m, max_slots=4, max_len=128, use_graphs=graphs)
        if graphs:
            eng.generate(prompts[:1], sp[:1])
        reqs = eng.generate(prompts, sp)
        outs.append([r.output for r in reqs])
    assert outs[0] == outs[1] == outs[2]


@pytest.mark.parametrize("device", ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)])
def test_beam_search_forks_the_state(device):
    m, w = make("loop", device, F32)
    eng = LLMEngine(m, max_slots=4, max_len=64, page_size=16)
    prompt = tokens(18, 131, 8)
    res = eng.beam_generate(prompt, 3, 5, len_penalty=0.0)
    ids = prompt + res.sequences[0]  # score of the returned sequence by the oracle
    lp = torch.log_softmax(bo.forward(CFGS["loop"][0], w, ids), -1)
    score = sum(float(lp[len(prompt) - 1 + i, t]) for i, t in enumerate(res.sequences[0]))
    assert abs(score - res.cum_logprobs[0]) < 1e-3
    assert len(eng.free) == 4


# ------------------------------------------------------------------------------- loading, replay, CLI
@pytest.mark.parametrize("name", list(CFGS))
def test_checkpoint_round_trip(tmp_path, name):
    """The bias tables' sizes come from the tensors, and stay through a save."""
    cfg, rows = CFGS[name]
    w = bo.random_weights(cfg, rows, 3)
    m = load_pretrained(write_dir(tmp_path / "a", cfg, w), dtype=BF16)
    assert m.cfg.arch == "begopel" and m.cfg.n_params() == m.num_parameters() >= sum(v.numel() for v in w.values())
    save_pretrained(m, str(tmp_path / "b"))
    from safetensors.torch import load_file
    back = load_file(str(tmp_path / "b" / "model.safetensors"))
    assert set(back) == set(w) and all(torch.equal(back[k].double(), w[k]) for k in w)
    m2 = load_pretrained(str(tmp_path / "b"), dtype=BF16)
    assert all(torch.equal(a, b) for a, b in zip(m.state_dict().values(), m2.state_dict().values()))


def test_loading_names_what_is_wrong(tmp_path):
    cfg, rows = CFGS["odd"]
    w = bo.random_weights(cfg, rows, 3)
    bad = dict(w)
    bad.pop("l1.mix.conv.b")
    with pytest.raises(RuntimeError, match="missing tensor l1.mix.conv.b"):
        load_pretrained(write_dir(tmp_path / "c", cfg, bad))
    with pytest.raises(RuntimeError, match="does not name"):
        load_pretrained(write_dir(tmp_path / "d", cfg, {**w, "l0.mix.left.extra": torch.zeros(1)}))
    with pytest.raises(ValueError, match="unknown mixer"):
        LMConfig.from_hf(config(16, 20, [({"type": "rnn", "mixer": {}}, None)]))
    c = copy.deepcopy(cfg)
    c["layers"][0]["mlp"]["kind"] = "moe"
    with pytest.raises(ValueError, match="unknown feed-forward"):
        LMConfig.from_hf(c)
    with pytest.raises(ValueError, match="equal parts"):
        LMConfig.from_hf(config(16, 20, [(ssd(2, 1, 8, 5, 2, 3), None)]))
    from kubernetes_cloud_amd.parallel.tensor_parallel import load_tp_model
    with pytest.raises(NotImplementedError, match="tensor parallelism.*begopel"):
        load_tp_model(write_dir(tmp_path / "m", cfg, w), 0, 1)
    with pytest.raises(TypeError, match="bf16 or fp32"):
        runner_of(build_model(LMConfig.from_hf(cfg), dtype=torch.float16))


def test_tensorized_round_trip(tmp_path):
    from kubernetes_cloud_amd.io.hf import load_tensorized, serialize_causal_lm
    m, _ = make("loop", "cpu", F32)
    serialize_causal_lm(m, str(tmp_path / "m.tensors"))
    m2, _ = load_tensorized(str(tmp_path / "m.tensors"), dtype=F32)
    ids = torch.tensor([tokens(9, 131, 1)])
    assert torch.equal(m(ids), m2(ids))


@pytest.mark.parametrize("device,dtype", WHERE)
def test_trace_replay(tmp_path, device, dtype):
    """The replay loop: files for steps that want logits, ``done`` after each, slots and pages given back."""
    from kubernetes_cloud_amd.engine import trace
    cfg, rows = CFGS["loop"]
    w = bo.random_weights(cfg, rows, 0)
    r = trace.open_runner(write_dir(tmp_path / "m", cfg, w), dtype, 190, device)
    assert r.cache.n_pages == 3 and r.max_slots == 4
    seqs = {i: tokens(n, cfg["vocab"], 80 + n) for i, n in (("p", 100), ("q", 30), ("r", 120))}
    steps = [[("p", 64, [63]), ("q", 2, [0, 1])], [("p", 1, [])], [("q", 28, [3]), ("p", 35, [34, 0])],
             [("r", 100, [99])], [("r", 20, [19])]]
    lines, at, want = [], dict.fromkeys(seqs, 0), {}
    for n, st in enumerate(steps):
        ent, end, logits = [], [], []
        for i, c, wn in st:
            ent.append({"id": i, "tokens": seqs[i][at[i]:at[i] + c], "want": wn})
            logits += [oracle("loop", w, seqs[i])[at[i] + k] for k in wn]
            at[i] += c
            if at[i] == len(seqs[i]):
                end.append(i)
        lines.append(json.dumps({"step": n, "entries": ent, "end": end}))
        want[n] = logits
    said = []
    trace.replay(r, lines, str(tmp_path), said.append)
    assert said == [f"done {n}" for n in range(5)]
    for n, logits in want.items():
        path = tmp_path / f"{n}.f32"
        assert path.exists() == bool(logits)
        if logits:
            got = torch.frombuffer(bytearray(path.read_bytes()), dtype=F32).view(len(logits), -1)
            close(got, torch.stack(logits), dtype)
    assert r.cache.free_count() == 3


def test_evaluator_takes_token_ids(tmp_path):
    from kubernetes_cloud_amd.train import evaluator
    cfg, rows = CFGS["plain"]
    w = bo.random_weights(cfg, rows, 0)
    path = write_dir(tmp_path / "m", cfg, w)
    prompt = [5, 17, 3, 77]
    if torch.cuda.is_available():
        pytest.skip("the CLI serves in bf16 on a GPU: ties decide")
    out = evaluator.main(["--model", path, "--prompt-ids", "5 17 3 77", "--prompt-tokens", "6", "--top-k", "1",
                          "--repetition-penalty", "1.0"])
    assert out["5 17 3 77"] == [" ".join(map(str, prompt + greedy("plain", w, prompt, 6)))]
