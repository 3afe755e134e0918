"""Rezusun: config.json reader and checkpoint names for ``models.hybrid_lm``.

Layers are listed one by one -- "latent_attention", "general_delta" or "channel_delta", each with its own sizes
and an optional gated feed-forward -- with layer norms before and after every sublayer, a layer scale, and a
range of layers that may run several times. The inner sizes of the two-step projections are the tensors'
(``with_shapes``); config.json may repeat them as "decay_rank" / "gate_rank".
"""
from __future__ import annotations

import copy
import dataclasses

import torch

from .hybrid_config import (ChannelDeltaSpec, GatedDenseSpec, GeneralDeltaSpec, HybridConfig, LatentAttentionSpec,
                            LayerSpec, LoopSpec)


def read_config(cfg: dict) -> HybridConfig:
    layers = []
    for i, L in enumerate(cfg["layers"]):
        mx, mlp, kind = L["mixer"], L.get("mlp"), L["type"]
        if kind == "latent_attention":
            rot = mx.get("rot") or {"base": 1.0, "dims": 0}
            mixer = LatentAttentionSpec(heads=mx["heads"], dim=mx["dim"], vdim=mx["vdim"], rot_dim=mx["rot_dim"],
                                        q_rank=mx["q_rank"], kv_rank=mx["kv_rank"], scale=mx["scale"],
                                        rot_base=rot["base"], rot_dims=rot["dims"])
        elif kind == "general_delta":
            mixer = GeneralDeltaSpec(heads=mx["heads"], dim=mx["dim"], decay_rank=mx.get("decay_rank"))
        elif kind == "channel_delta":
            mixer = ChannelDeltaSpec(heads=mx["heads"], kv_heads=mx["kv_heads"], dim=mx["dim"], vdim=mx["vdim"],
                                     taps=mx["conv"], decay_rank=mx.get("decay_rank"), gate_rank=mx.get("gate_rank"))
        else:
            raise ValueError(f"layer {i}: unknown mixer type {kind!r} (latent_attention, general_delta, channel_delta)")
        if mlp is None:
            ff = None
        elif mlp["kind"] == "dense":
            ff = GatedDenseSpec(ff=mlp["ff"])
        else:
            raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r} (dense)")
        layers.append(LayerSpec(mixer, ff))
    lp = cfg.get("loop")
    out = HybridConfig(arch="rezusun", vocab_size=cfg["vocab"], hidden=cfg["width"], layers=tuple(layers),
                       norm_eps=cfg["norm"]["eps"], block="sandwich",
                       loop=LoopSpec(lp["start"], lp["stop"], lp["times"]) if lp else None, hf=cfg)
    out.runs  # (a range outside the layers raises here)
    return out


def with_shapes(cfg: HybridConfig, shapes: dict) -> HybridConfig:
    """``cfg`` with the inner sizes that the tensors' shapes give."""
    hf = copy.deepcopy(cfg.hf)
    layers = []
    for i, L in enumerate(cfg.layers):
        ranks = {k: shapes[f"l{i}.mix.{t}"][0] for k, t in _RANKS.get(type(L.mixer), {}).items() if f"l{i}.mix.{t}" in shapes}
        hf["layers"][i]["mixer"].update(ranks)
        layers.append(LayerSpec(dataclasses.replace(L.mixer, **ranks), L.mlp))
    return dataclasses.replace(cfg, layers=tuple(layers), hf=hf)


_RANKS = {GeneralDeltaSpec: {"decay_rank": "w1"}, ChannelDeltaSpec: {"decay_rank": "a1", "gate_rank": "g1"}}
# module parameter -> checkpoint tensor under "l<i>.mix."
_EXTRA = {
    LatentAttentionSpec: {"q_norm": "dq.norm", "kv_norm": "dkv.norm", "uq": "uq", "sink": "sink"},
    GeneralDeltaSpec: {"w2": "w2", "w0": "w0", "a_bias": "a.b", "gain": "norm"},
    ChannelDeltaSpec: {"a2": "a2", "dt_bias": "dt_bias", "a_log": "A_log", "g2": "g2", "gain": "norm"},
}


def to_native(sd: dict, cfg: HybridConfig) -> dict:
    """Checkpoint tensors -> ``HybridLM`` parameters. Missing and left-over names raise."""
    left, out = set(sd), {}

    def take(name):
        if name not in sd:
            raise RuntimeError(f"missing tensor {name}")
        left.discard(name)
        return sd[name]

    out["wte"], out["head"], out["final_norm"] = take("embed"), take("head"), take("final.norm")
    for i, L in enumerate(cfg.layers):
        s, n, mx = f"l{i}.", f"layers.{i}.", L.mixer
        m = s + "mix."
        out[n + "norm"], out[n + "norm_b"], out[n + "scale"] = take(s + "norm1"), take(s + "norm1b"), take(s + "ls1")
        first = sd[m + next(iter(mx.parts))]
        w_in = first.new_zeros(mx.in_rows, cfg.hidden)
        for name, (o, size) in mx.parts.items():
            w_in[o:o + size] = take(m + name)
        out[n + "w_in"], out[n + "w_out"] = w_in, take(m + "o")
        for p, name in _EXTRA[type(mx)].items():
            out[n + p] = take(m + name)
        if isinstance(mx, LatentAttentionSpec):
            out[n + "ukv"] = torch.cat([take(m + "uk"), take(m + "uv")])
        elif isinstance(mx, ChannelDeltaSpec):
            out[n + "conv"] = torch.cat([take(m + x + ".conv") for x in "qkv"])
        if L.mlp is not None:
            q = s + "mlp."
            out[n + "norm2"], out[n + "norm2_b"], out[n + "scale2"] = take(s + "norm2"), take(s + "norm2b"), take(s + "ls2")
            out[n + "w_up"] = torch.cat([take(q + "gate"), take(q + "up")])
            out[n + "b_up"] = torch.cat([take(q + "gate.b"), take(q + "up.b")])
            out[n + "w_down"], out[n + "b_down"] = take(q + "down"), take(q + "down.b")
    if left:
        raise RuntimeError(f"tensors the configuration does not name: {sorted(left)[:8]}")
    return out


def from_native(sd: dict, cfg: HybridConfig) -> dict:
    """``HybridLM`` parameters -> checkpoint tensors."""
    out = {"embed": sd["wte"], "head": sd["head"], "final.norm": sd["final_norm"]}
    for i, L in enumerate(cfg.layers):
        s, n, mx = f"l{i}.", f"layers.{i}.", L.mixer
        m = s + "mix."
        out[s + "norm1"], out[s + "norm1b"], out[s + "ls1"] = sd[n + "norm"], sd[n + "norm_b"], sd[n + "scale"]
        for name, (o, size) in mx.parts.items():
            out[m + name] = sd[n + "w_in"][o:o + size]
        out[m + "o"] = sd[n + "w_out"]
        for p, name in _EXTRA[type(mx)].items():
            out[m + name] = sd[n + p]
        if isinstance(mx, LatentAttentionSpec):
            out[m + "uk"], out[m + "uv"] = sd[n + "ukv"].split([mx.heads * mx.dim, mx.heads * mx.vdim])
        elif isinstance(mx, ChannelDeltaSpec):
            nk = mx.kv_heads * mx.dim
            for x, t in zip("qkv", sd[n + "conv"].split([nk, nk, mx.heads * mx.vdim])):
                out[m + x + ".conv"] = t
        if L.mlp is not None:
            q = s + "mlp."
            out[s + "norm2"], out[s + "norm2b"], out[s + "ls2"] = sd[n + "norm2"], sd[n + "norm2_b"], sd[n + "scale2"]
            out[q + "gate"], out[q + "up"] = sd[n + "w_up"].chunk(2)
            out[q + "gate.b"], out[q + "up.b"] = sd[n + "b_up"].chunk(2)
            out[q + "down"], out[q + "down.b"] = sd[n + "w_down"], sd[n + "b_down"]
    return out


__all__ = ["read_config", "with_shapes", "to_native", "from_native"]
