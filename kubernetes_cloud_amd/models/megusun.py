"""Megusun: config.json reader and checkpoint names for ``models.hybrid_lm``.

Layers are listed one by one ("attention": differential attention, "mingru": gated recurrence), each with its
own sizes and feed-forward; one RMS norm (a single number) feeds both branches, and a token shift precedes
the mixer.
"""
from __future__ import annotations

import torch

from .hybrid_config import (DenseSpec, DiffAttentionSpec, GatedRecurrenceSpec, HybridConfig, LayerSpec, MoESpec)


def read_config(cfg: dict) -> HybridConfig:
    layers = []
    for i, L in enumerate(cfg["layers"]):
        mx, mlp = L["mixer"], L.get("mlp")
        if L["type"] == "attention":
            qt = mx.get("q_temp") or {}
            mixer = DiffAttentionSpec(heads=mx["heads"], kv_heads=mx["kv_heads"], dim=mx["dim"], vdim=mx["vdim"],
                                      scale=mx["scale"], diff=mx["diff"], temp_coef=qt.get("coef", 0.0),
                                      temp_every=qt.get("every", 0.0))
        elif L["type"] == "mingru":
            mixer = GatedRecurrenceSpec(width=mx["width"])
        else:
            raise ValueError(f"layer {i}: unknown mixer type {L['type']!r} (attention, mingru)")
        if mlp is None:
            ff = None
        elif mlp["kind"] == "dense":
            ff = DenseSpec(ff=mlp["ff"])
        elif mlp["kind"] == "moe":
            ff = MoESpec(experts=mlp["router"]["experts"], top=mlp["router"]["top"], ff=mlp["expert"]["ff"],
                         shared_ff=(mlp.get("shared") or {}).get("ff", 0))
        else:
            raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r} (dense, moe)")
        layers.append(LayerSpec(mixer, ff))
    return HybridConfig(arch="megusun", vocab_size=cfg["vocab"], hidden=cfg["width"], layers=tuple(layers),
                        norm_eps=cfg["norm"]["eps"], residual_mult=cfg["residual_mult"], hf=cfg)


def _mixer_in(spec) -> tuple:
    return ("q", "k", "v") if isinstance(spec.mixer, DiffAttentionSpec) else ("z", "x", "g")


def to_native(sd: dict, cfg: HybridConfig) -> dict:
    """Checkpoint tensors -> ``HybridLM`` parameters. Missing and left-over names raise."""
    left, out = set(sd), {}

    def take(name):
        if name not in sd:
            raise RuntimeError(f"missing tensor {name}")
        left.discard(name)
        return sd[name]

    out["wte"], out["head"], out["final_norm"] = take("embed"), take("head"), take("final.norm").reshape(())
    for i, L in enumerate(cfg.layers):
        s, n = f"l{i}.", f"layers.{i}."
        out[n + "norm"], out[n + "shift"] = take(s + "norm1").reshape(()), take(s + "shift")
        out[n + "w_in"] = torch.cat([take(s + "mix." + x) for x in _mixer_in(L)])
        if isinstance(L.mixer, DiffAttentionSpec):
            out[n + "lam"] = torch.stack([take(s + "mix." + x) for x in ("lq1", "lk1", "lq2", "lk2")])
        else:
            out[n + "b_z"], out[n + "b_x"] = take(s + "mix.z.b"), take(s + "mix.x.b")
        w_out = [take(s + "mix.o")]
        if isinstance(L.mlp, DenseSpec):
            out[n + "w_up"] = take(s + "mlp.up")
            w_out.append(take(s + "mlp.down"))
        elif isinstance(L.mlp, MoESpec):
            e = [f"{s}mlp.e{j}." for j in range(L.mlp.experts)]
            out[n + "router"] = take(s + "mlp.router")
            out[n + "gate_up"] = torch.stack([torch.cat([take(x + "gate"), take(x + "up")]) for x in e])
            out[n + "down"] = torch.stack([take(x + "down") for x in e])
            if L.mlp.shared_ff:
                q = s + "mlp.shared."
                out[n + "w_up"] = torch.cat([take(q + "gate"), take(q + "up")])
                out[n + "shared_gate"] = take(q + "sg").reshape(1, -1)
                w_out.append(take(q + "down"))
        out[n + "w_out"] = torch.cat(w_out, dim=1)
    if left:
        raise RuntimeError(f"tensors the configuration does not name: {sorted(left)[:8]}")
    return out


def from_native(sd: dict, cfg: HybridConfig) -> dict:
    """``HybridLM`` parameters -> checkpoint tensors."""
    out = {"embed": sd["wte"], "head": sd["head"], "final.norm": sd["final_norm"]}
    for i, L in enumerate(cfg.layers):
        s, n, mx = f"l{i}.", f"layers.{i}.", L.mixer
        out[s + "norm1"], out[s + "shift"] = sd[n + "norm"], sd[n + "shift"]
        attn = isinstance(mx, DiffAttentionSpec)
        sizes = ([2 * mx.heads * mx.dim, 2 * mx.kv_heads * mx.dim, mx.kv_heads * mx.vdim] if attn
                 else [mx.width] * 3)
        for name, t in zip(_mixer_in(L), sd[n + "w_in"].split(sizes)):
            out[s + "mix." + name] = t
        if attn:
            for name, t in zip(("lq1", "lk1", "lq2", "lk2"), sd[n + "lam"]):
                out[s + "mix." + name] = t
        else:
            out[s + "mix.z.b"], out[s + "mix.x.b"] = sd[n + "b_z"], sd[n + "b_x"]
        out[s + "mix.o"] = sd[n + "w_out"][:, :mx.out_cols]
        tail = sd[n + "w_out"][:, mx.out_cols:]
        if isinstance(L.mlp, DenseSpec):
            out[s + "mlp.up"], out[s + "mlp.down"] = sd[n + "w_up"], tail
        elif isinstance(L.mlp, MoESpec):
            out[s + "mlp.router"] = sd[n + "router"]
            for j in range(L.mlp.experts):
                q = f"{s}mlp.e{j}."
                out[q + "gate"], out[q + "up"] = sd[n + "gate_up"][j].chunk(2)
                out[q + "down"] = sd[n + "down"][j]
            if L.mlp.shared_ff:
                q = s + "mlp.shared."
                out[q + "gate"], out[q + "up"] = sd[n + "w_up"].chunk(2)
                out[q + "sg"], out[q + "down"] = sd[n + "shared_gate"], tail
    return out


__all__ = ["read_config", "to_native", "from_native"]
