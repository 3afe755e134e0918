"""Gibipel: config.json reader and checkpoint names for ``models.hybrid_lm``.

Layers are listed one by one, each with its own sizes: two mixers of the same rows side by side -- sliding-window
attention that sees what lies before its window as block means, and a matrix memory (mLSTM) -- joined by fixed
weights, then routed experts with a shared one, or no feed-forward. Both sublayers read the stream itself; what they add
is RMS-normed with one gain. The embedding is scaled, the output projection a matrix of its own.
"""
from __future__ import annotations

import torch

from .hybrid_config import HybridConfig, LayerSpec, MatrixMemorySpec, MoESpec, PooledAttentionSpec, SumSpec


def _mixer(mx: dict) -> SumSpec:
    a, b = mx["left"], mx["right"]
    rot, mask = a["rot"], a["mask"]
    sc = rot.get("scaling")
    return SumSpec(
        PooledAttentionSpec(heads=a["heads"], kv_heads=a["kv_heads"], dim=a["dim"], vdim=a["vdim"], scale=a["scale"],
                            window=mask["size"], pool=mask["pool"], rot_base=rot["base"], rot_dims=rot["dims"],
                            rot_scaling=None if sc is None else (sc["factor"], sc["low"], sc["high"], sc["original"])),
        MatrixMemorySpec(heads=b["heads"], dim=b["dim"], vdim=b["vdim"], gate_cap=b["gate_cap"]),
        mx["left_scale"], mx["right_scale"])


def _routed(mlp: dict) -> MoESpec:
    r = mlp["router"]
    groups, shared = r.get("groups") or {"count": 1, "keep": 1}, mlp.get("shared")
    return MoESpec(experts=r["experts"], top=r["top"], ff=mlp["expert"]["ff"], shared_ff=shared["ff"] if shared else 0,
                   scale_in=False, shared_gate=False, score="softmax", identity=r.get("identity") or 0,
                   groups=groups["count"], keep=groups["keep"], correction=True)


def read_config(cfg: dict) -> HybridConfig:
    layers = []
    for i, L in enumerate(cfg["layers"]):
        mlp = L.get("mlp")
        if L["type"] != "parallel":
            raise ValueError(f"layer {i}: unknown mixer type {L['type']!r} (parallel)")
        if mlp is not None and mlp["kind"] != "moe":
            raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r} (moe)")
        layers.append(LayerSpec(_mixer(L["mixer"]), None if mlp is None else _routed(mlp)))
    return HybridConfig(arch="gibipel", vocab_size=cfg["vocab"], hidden=cfg["width"], layers=tuple(layers),
                        norm_eps=cfg["norm"]["eps"], block="postnorm", embed_scale=cfg["embedding"]["scale"],
                        logit_scale=cfg["logit_scale"], hf=cfg)


# module parameter -> checkpoint tensor under the mixer's prefix
_LEFT = {"q_norm": "q.norm", "k_norm": "k.norm", "sink": "sink"}
_RIGHT = {"i_bias": "i.b", "f_bias": "f.b", "gain": "norm"}


def _blocks(mx: SumSpec) -> list:
    """(checkpoint tensor under the mixer, its first row of ``w_in``, rows) of both sides."""
    out = []
    for side, spec, base in (("left.", mx.left, 0), ("right.", mx.right, mx.left.in_rows)):
        out += [(side + name, base + o, n) for name, (o, n) in spec.parts.items()]
    return out


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
        s, n, mx, mlp = f"l{i}.", f"layers.{i}.", L.mixer, L.mlp
        m, f = s + "mix.", s + "mlp."
        out[n + "norm"] = take(s + "norm1")
        w_in = out[n + "w_in"] = out["wte"].new_zeros(mx.in_rows, cfg.hidden)
        b_in = out[n + "b_in"] = out["wte"].new_zeros(mx.in_rows)
        for name, o, size in _blocks(mx):
            w_in[o:o + size] = take(m + name)
            if name.startswith("left."):
                b_in[o:o + size] = take(m + name + ".b")
        w_out = out[n + "w_out"] = out["wte"].new_zeros(cfg.hidden, mx.out_cols)
        for side, names, (o, size) in zip(("left.", "right."), (_LEFT, _RIGHT), mx.out_parts.values()):
            out.update((n + side + p, take(m + side + name)) for p, name in names.items())
            w_out[:, o:o + size] = take(m + side + "o")
        if mlp is None:
            continue
        out[n + "norm2"], out[n + "router"], out[n + "correction"] = take(s + "norm2"), take(f + "router"), take(f + "correction")
        out[n + "gate_up"] = torch.stack([torch.cat([take(f"{f}e{e}.gate"), take(f"{f}e{e}.up")]) for e in range(mlp.experts)])
        out[n + "down"] = torch.stack([take(f"{f}e{e}.down") for e in range(mlp.experts)])
        if mlp.shared_ff:
            out[n + "w_up"] = torch.cat([take(f + "shared.gate"), take(f + "shared.up")])
            out[n + "w_down"] = take(f + "shared.down")
    if left:
        raise RuntimeError(f"tensors the configuration does not name: {sorted(left)[:8]}")
    return out


def from_native(sd: dict, cfg: HybridConfig) -> dict:
    """``HybridLM`` parameters -> checkpoint tensors."""
    out = {"embed": sd["wte"], "head": sd["head"], "final.norm": sd["final_norm"]}
    for i, L in enumerate(cfg.layers):
        s, n, mx, mlp = f"l{i}.", f"layers.{i}.", L.mixer, L.mlp
        m, f = s + "mix.", s + "mlp."
        out[s + "norm1"] = sd[n + "norm"]
        for name, o, size in _blocks(mx):
            out[m + name] = sd[n + "w_in"][o:o + size]
            if name.startswith("left."):
                out[m + name + ".b"] = sd[n + "b_in"][o:o + size]
        for side, names, (o, size) in zip(("left.", "right."), (_LEFT, _RIGHT), mx.out_parts.values()):
            out.update((m + side + name, sd[n + side + p]) for p, name in names.items())
            out[m + side + "o"] = sd[n + "w_out"][:, o:o + size]
        if mlp is None:
            continue
        out[s + "norm2"], out[f + "router"], out[f + "correction"] = sd[n + "norm2"], sd[n + "router"], sd[n + "correction"]
        for e in range(mlp.experts):
            out[f"{f}e{e}.gate"], out[f"{f}e{e}.up"] = sd[n + "gate_up"][e].split(mlp.ff)
            out[f"{f}e{e}.down"] = sd[n + "down"][e]
        if mlp.shared_ff:
            out[f + "shared.gate"], out[f + "shared.up"] = sd[n + "w_up"].split(mlp.shared_ff)
            out[f + "shared.down"] = sd[n + "w_down"]
    return out


__all__ = ["read_config", "to_native", "from_native"]
