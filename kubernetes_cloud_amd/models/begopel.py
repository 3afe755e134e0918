"""Begopel: config.json reader and checkpoint names for ``models.hybrid_lm``.

Layers are listed one by one -- "mamba2" (a selective state space) or "parallel" (biased attention and a gated delta
rule side by side), each with its own sizes and an optional squared-ReLU feed-forward -- with RMS norms before every
sublayer. A range of layers may run several times, each pass entered through a projection of the stream and the
embedding output. The embedding table is the output projection; logits are soft-capped. The rows of the bias tables
are the tensors' (``with_shapes``); config.json may repeat them as "bias_rows".
"""
from __future__ import annotations

import copy
import dataclasses

import torch

from .hybrid_config import (BiasedAttentionSpec, DenseSpec, HeadDeltaSpec, HybridConfig, LayerSpec, LoopSpec,
                            SideBySideSpec, SsdSpec)


def _side_by_side(mx: dict) -> SideBySideSpec:
    a, b = mx["left"], mx["right"]
    rows = {"bias_rows": a["bias_rows"]} if "bias_rows" in a else {}
    return SideBySideSpec(
        BiasedAttentionSpec(heads=a["heads"], kv_heads=a["kv_heads"], dim=a["dim"], vdim=a["vdim"], scale=a["scale"],
                            bias_max=a["bias_max"], **rows),
        HeadDeltaSpec(heads=b["heads"], kv_heads=b["kv_heads"], dim=b["dim"], vdim=b["vdim"], taps=b["conv"]))


def read_config(cfg: dict) -> HybridConfig:
    layers = []
    for i, L in enumerate(cfg["layers"]):
        mx, mlp, kind = L["mixer"], L.get("mlp"), L["type"]
        if kind == "parallel":
            mixer = _side_by_side(mx)
        elif kind == "mamba2":
            mixer = SsdSpec(heads=mx["heads"], groups=mx["groups"], state=mx["state"], vdim=mx["vdim"], taps=mx["conv"],
                            norm_groups=mx["norm_groups"])
        else:
            raise ValueError(f"layer {i}: unknown mixer type {kind!r} (mamba2, parallel)")
        if mlp is None:
            ff = None
        elif mlp["kind"] == "dense":
            ff = DenseSpec(ff=mlp["ff"], act="relu2")
        else:
            raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r} (dense)")
        layers.append(LayerSpec(mixer, ff))
    lp = cfg.get("loop")
    out = HybridConfig(arch="begopel", vocab_size=cfg["vocab"], hidden=cfg["width"], layers=tuple(layers),
                       norm_eps=cfg["norm"]["eps"], block="prenorm", embed_scale=cfg["embedding"]["scale"], tied=True,
                       logit_softcap=cfg.get("logit_softcap") or 0.0,
                       loop=LoopSpec(lp["start"], lp["stop"], lp["times"], entry=True) if lp else None, hf=cfg)
    out.runs  # (a range outside the layers raises here)
    return out


def with_shapes(cfg: HybridConfig, shapes: dict) -> HybridConfig:
    """``cfg`` with the bias table sizes that the tensors' shapes give."""
    hf = copy.deepcopy(cfg.hf)
    layers = []
    for i, L in enumerate(cfg.layers):
        name = f"l{i}.mix.left.rel"
        if isinstance(L.mixer, SideBySideSpec) and name in shapes:
            rows = shapes[name][0]
            hf["layers"][i]["mixer"]["left"]["bias_rows"] = rows
            L = LayerSpec(dataclasses.replace(L.mixer, left=dataclasses.replace(L.mixer.left, bias_rows=rows)), L.mlp)
        layers.append(L)
    return dataclasses.replace(cfg, layers=tuple(layers), hf=hf)


# module parameter -> checkpoint tensor under the mixer's prefix
_EXTRA = {
    BiasedAttentionSpec: {"q_norm": "q.norm", "k_norm": "k.norm", "rel": "rel", "sink": "sink"},
    HeadDeltaSpec: {"dt_bias": "dt_bias", "a_log": "A_log", "gain": "norm"},
    SsdSpec: {"dt_bias": "dt_bias", "a_log": "A_log", "skip": "D", "gain": "norm"},
}
_SIDE = {"w_out": "o", "out_norm": "out"}


def _ssd_blocks(mx: SsdSpec) -> list:
    """Row blocks of the checkpoint's input projection, in its order."""
    n, s = mx.out_cols, mx.groups * mx.state
    return [("z", n), ("x", n), ("B", s), ("C", s), ("dt", mx.heads)]


def _conv_to_native(t, mx: SsdSpec):
    x, b, c = t.split([mx.out_cols, mx.groups * mx.state, mx.groups * mx.state])
    return torch.cat([c, b, x])


def _conv_from_native(t, mx: SsdSpec):
    c, b, x = t.split([mx.groups * mx.state, mx.groups * mx.state, mx.out_cols])
    return torch.cat([x, b, c])


def to_native(sd: dict, cfg: HybridConfig) -> dict:
    """Checkpoint tensors -> ``HybridLM`` parameters. Missing and left-over names raise."""
    left, out = set(sd), {}

    def take(name):
        if name not in sd:
            raise RuntimeError(f"missing tensor {name}")
        left.discard(name)
        return sd[name]

    def side(m, n, mx, w_in):
        for name, (o, size) in mx.parts.items():
            w_in[o:o + size] = take(m + name)
        for p, name in {**_EXTRA[type(mx)], **_SIDE}.items():
            out[n + p] = take(m + name)
        if isinstance(mx, HeadDeltaSpec):
            out[n + "conv"] = torch.cat([take(m + x + ".conv") for x in "qkv"])

    out["wte"], out["final_norm"] = take("embed"), take("final.norm")
    if cfg.loop is not None:
        out["loop_in"], out["loop_step"] = take("loop.in"), take("loop.step")
    for i, L in enumerate(cfg.layers):
        s, n, mx = f"l{i}.", f"layers.{i}.", L.mixer
        m = s + "mix."
        out[n + "norm"] = take(s + "norm1")
        w_in = out[n + "w_in"] = out[n + "norm"].new_zeros(mx.in_rows, cfg.hidden)
        if isinstance(mx, SideBySideSpec):
            side(m + "left.", n + "left.", mx.left, w_in)
            side(m + "right.", n + "right.", mx.right, w_in[mx.in_rows - mx.right.in_rows:])
        else:
            for (name, size), rows in zip(_ssd_blocks(mx), take(m + "in").split([b for _, b in _ssd_blocks(mx)])):
                w_in[mx.parts[name][0]:mx.parts[name][0] + size] = rows
            for p, name in _EXTRA[SsdSpec].items():
                out[n + p] = take(m + name)
            out[n + "conv"], out[n + "conv_b"] = (_conv_to_native(take(m + x), mx) for x in ("conv", "conv.b"))
            out[n + "w_out"] = take(m + "o")
        if L.mlp is not None:
            out[n + "norm2"], out[n + "w_up"], out[n + "w_down"] = take(s + "norm2"), take(s + "mlp.up"), take(s + "mlp.down")
    if left:
        raise RuntimeError(f"tensors the configuration does not name: {sorted(left)[:8]}")
    return out


def from_native(sd: dict, cfg: HybridConfig) -> dict:
    """``HybridLM`` parameters -> checkpoint tensors."""
    out = {"embed": sd["wte"], "final.norm": sd["final_norm"]}

    def side(m, n, mx, w_in):
        for name, (o, size) in mx.parts.items():
            out[m + name] = w_in[o:o + size]
        for p, name in {**_EXTRA[type(mx)], **_SIDE}.items():
            out[m + name] = sd[n + p]
        if isinstance(mx, HeadDeltaSpec):
            nk = mx.kv_heads * mx.dim
            for x, t in zip("qkv", sd[n + "conv"].split([nk, nk, mx.out_cols])):
                out[m + x + ".conv"] = t

    if cfg.loop is not None:
        out["loop.in"], out["loop.step"] = sd["loop_in"], sd["loop_step"]
    for i, L in enumerate(cfg.layers):
        s, n, mx = f"l{i}.", f"layers.{i}.", L.mixer
        m, w_in = s + "mix.", sd[n + "w_in"]
        out[s + "norm1"] = sd[n + "norm"]
        if isinstance(mx, SideBySideSpec):
            side(m + "left.", n + "left.", mx.left, w_in)
            side(m + "right.", n + "right.", mx.right, w_in[mx.in_rows - mx.right.in_rows:])
        else:
            out[m + "in"] = torch.cat([w_in[mx.parts[k][0]:mx.parts[k][0] + size] for k, size in _ssd_blocks(mx)])
            for p, name in _EXTRA[SsdSpec].items():
                out[m + name] = sd[n + p]
            out[m + "conv"], out[m + "conv.b"] = (_conv_from_native(sd[n + x], mx) for x in ("conv", "conv_b"))
            out[m + "o"] = sd[n + "w_out"]
        if L.mlp is not None:
            out[s + "norm2"], out[s + "mlp.up"], out[s + "mlp.down"] = sd[n + "norm2"], sd[n + "w_up"], sd[n + "w_down"]
    return out


__all__ = ["read_config", "with_shapes", "to_native", "from_native"]
