"""Plain, slow Begopel forward used as the oracle of the Begopel tests: whole sequences, one function per
mechanism, a loop over tokens wherever a recurrence is the definition, float64. It shares no code with the
product path.

``weights`` is a dict of float64 tensors under the checkpoint's tensor names, ``cfg`` the parsed config.json.
"""
import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_about_one(x, w, eps):
    """RMS norm whose gain is 1 + w."""
    return rms(x, eps) * (1 + w)


def unit(x):
    """Unit vectors, with 1e-6 under the root."""
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.log1p(torch.exp(-z.abs())) + torch.clamp(z, min=0)


def causal_conv(x, taps):
    """Per-channel convolution over time, the last tap on the current row, zeros before the start."""
    T, n = x.shape[0], taps.shape[1]
    out = torch.zeros_like(x)
    for t in range(T):
        for i in range(n):
            if t - i >= 0:
                out[t] += taps[:, n - 1 - i] * x[t - i]
    return out


def distance_bucket(n, rows, far):
    """Row of the bias table for distance n: one each for the near half, then evenly spaced in ln(distance)
    up to ``far``, the last row beyond."""
    near = rows / 2
    if n < near:
        return n
    return min(rows - 1, int(near + math.floor(math.log(n / near) / math.log(far / near) * (rows - near))))


def sink_softmax_row(scores, sink):
    """exp(s_j) / (exp(sink) + sum_j exp(s_j))."""
    m = max(float(scores.max()), float(sink))
    e = torch.exp(scores - m)
    return e / (e.sum() + math.exp(float(sink) - m))


def biased_attention(h, w, p, mx, eps):
    """Causal attention with normed queries and keys, a bias by bucketed distance, a sink, and a gate on the
    heads' outputs."""
    H, G, D, E = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    T = h.shape[0]
    q = rms((h @ w[p + "q"].T).view(T, H, D), eps) * w[p + "q.norm"]
    k = rms((h @ w[p + "k"].T).view(T, G, D), eps) * w[p + "k.norm"]
    v = (h @ w[p + "v"].T).view(T, G, E)
    table = w[p + "rel"]
    bias = torch.stack([table[distance_bucket(n, table.shape[0], mx["bias_max"])] for n in range(T)])  # [distance, H]
    out = torch.empty(T, H, E, dtype=h.dtype)
    for t in range(T):
        for a in range(H):
            g = a // (H // G)
            s = (k[:t + 1, g] @ q[t, a]) * mx["scale"] + bias[:t + 1, a].flip(0)
            out[t, a] = sink_softmax_row(s, w[p + "sink"][a]) @ v[:t + 1, g]
    return (out.reshape(T, H * E) * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def head_delta(h, w, p, mx, eps):
    """S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q, with one decay per head and token."""
    H, G, D, E = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    T = h.shape[0]
    q, k, v = (silu(causal_conv(h @ w[p + n].T, w[p + n + ".conv"])) for n in ("q", "k", "v"))
    q = unit(q.view(T, G, D)) * D ** -0.5
    k = unit(k.view(T, G, D))
    v = v.view(T, H, E)
    beta = torch.sigmoid(h @ w[p + "b"].T)
    g = torch.exp(-torch.exp(w[p + "A_log"]) * softplus(h @ w[p + "a"].T + w[p + "dt_bias"]))
    o = torch.empty(T, H, E, dtype=h.dtype)
    for i in range(H):
        S, j = torch.zeros(D, E, dtype=h.dtype), i // (H // G)
        for t in range(T):
            S = g[t, i] * S
            S = S + torch.outer(k[t, j], beta[t, i] * (v[t, i] - k[t, j] @ S))
            o[t, i] = q[t, j] @ S
    gate = silu(h @ w[p + "g"].T).view(T, H, E)
    return (rms(o, eps) * w[p + "norm"] * gate).reshape(T, H * E) @ w[p + "o"].T


def side_by_side(h, w, p, mx, eps):
    """Half the sum of two mixers' outputs, each normed over the model width."""
    a = rms(biased_attention(h, w, p + "left.", mx["left"], eps), eps) * w[p + "left.out"]
    b = rms(head_delta(h, w, p + "right.", mx["right"], eps), eps) * w[p + "right.out"]
    return (a + b) / 2


def ssd(h, w, p, mx, eps):
    """S <- exp(-exp(A) dt) S + dt B x^T, y = S^T C + D x per head; gated, then normed in equal parts."""
    H, E, N, G = mx["heads"], mx["vdim"], mx["state"], mx["groups"]
    T, n = h.shape[0], H * E
    z, c, dt = (h @ w[p + "in"].T).split([n, n + 2 * G * N, H], -1)
    c = silu(causal_conv(c, w[p + "conv"]) + w[p + "conv.b"])
    x, B, C = c[:, :n].view(T, H, E), c[:, n:n + G * N].view(T, G, N), c[:, n + G * N:].view(T, G, N)
    dt = softplus(dt + w[p + "dt_bias"])
    y = torch.empty(T, H, E, dtype=h.dtype)
    for i in range(H):
        S, j = torch.zeros(N, E, dtype=h.dtype), i // (H // G)
        for t in range(T):
            S = torch.exp(-torch.exp(w[p + "A_log"][i]) * dt[t, i]) * S + dt[t, i] * torch.outer(B[t, j], x[t, i])
            y[t, i] = C[t, j] @ S + w[p + "D"][i] * x[t, i]
    y = y.reshape(T, n) * silu(z)
    return (rms(y.view(T, mx["norm_groups"], -1), eps).reshape(T, n) * w[p + "norm"]) @ w[p + "o"].T


MIXERS = {"parallel": side_by_side, "mamba2": ssd}


def feed_forward(h, w, p):
    return torch.relu(h @ w[p + "up"].T) ** 2 @ w[p + "down"].T


def softcap(z, cap):
    return cap * torch.tanh(z / cap)


def order(cfg):
    """(layer, pass it opens or None) as they run: the looped range several times in a row."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, None) for i in range(n)]
    a, b = lp["start"], lp["stop"]
    loop = [(i, t if i == a else None) for t in range(lp["times"]) for i in range(a, b)]
    return [(i, None) for i in range(a)] + loop + [(i, None) for i in range(b, n)]


def forward(cfg, weights, tokens, layers_out=None):
    """Logits [T, vocab] of one whole sequence. ``layers_out`` collects the residual stream after every run."""
    w, eps = weights, cfg["norm"]["eps"]
    x0 = x = w["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
    for i, opens in order(cfg):
        L, s = cfg["layers"][i], f"l{i}."
        if opens is not None:
            x = torch.cat([x, x0], -1) @ w["loop.in"].T + w["loop.step"][opens]
        x = x + MIXERS[L["type"]](rms_about_one(x, w[s + "norm1"], eps), w, s + "mix.", L["mixer"], eps)
        if L["mlp"] is not None:
            x = x + feed_forward(rms_about_one(x, w[s + "norm2"], eps), w, s + "mlp.")
        if layers_out is not None:
            layers_out.append(x.clone())
    return softcap(rms_about_one(x, w["final.norm"], eps) @ w["embed"].T, cfg["logit_softcap"])


def tensor_shapes(cfg, rel_rows):
    """Checkpoint names -> shapes; ``rel_rows``: {layer: rows of its bias table}."""
    d, V, out = cfg["width"], cfg["vocab"], {}
    out.update({"embed": (V, d), "final.norm": (d,)})
    if cfg.get("loop"):
        out.update({"loop.in": (d, 2 * d), "loop.step": (cfg["loop"]["times"], d)})
    for i, L in enumerate(cfg["layers"]):
        s, mx = f"l{i}.", L["mixer"]
        m = s + "mix."
        out[s + "norm1"] = (d,)
        if L["type"] == "mamba2":
            H, E, N, G = (mx[k] for k in ("heads", "vdim", "state", "groups"))
            c = H * E + 2 * G * N
            out.update({m + "in": (H * E + c + H, d), m + "conv": (c, mx["conv"]), m + "conv.b": (c,), m + "dt_bias": (H,),
                        m + "A_log": (H,), m + "D": (H,), m + "norm": (H * E,), m + "o": (d, H * E)})
        else:
            a, b = mx["left"], mx["right"]
            H, G, D, E = (a[k] for k in ("heads", "kv_heads", "dim", "vdim"))
            l = m + "left."
            out.update({l + "q": (H * D, d), l + "k": (G * D, d), l + "v": (G * E, d), l + "q.norm": (D,), l + "k.norm": (D,),
                        l + "rel": (rel_rows[i], H), l + "sink": (H,), l + "g": (H * E, d), l + "o": (d, H * E), l + "out": (d,)})
            H, G, D, E = (b[k] for k in ("heads", "kv_heads", "dim", "vdim"))
            r = m + "right."
            for k, c in (("q", G * D), ("k", G * D), ("v", H * E)):
                out.update({r + k: (c, d), r + k + ".conv": (c, b["conv"])})
            out.update({r + "b": (H, d), r + "A_log": (H,), r + "norm": (E,), r + "a": (H, d), r + "dt_bias": (H,),
                        r + "g": (H * E, d), r + "o": (d, H * E), r + "out": (d,)})
        if L["mlp"] is not None:
            f = L["mlp"]["ff"]
            out.update({s + "norm2": (d,), s + "mlp.up": (f, d), s + "mlp.down": (d, f)})
    return out


def random_weights(cfg, rel_rows, seed=0):
    """Random float64 weights that bf16 holds exactly; decays from slow to fast, visible sinks and biases."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg, rel_rows).items():
        z = torch.randn(*shape, generator=g)
        leaf = name.rsplit(".", 1)[-1]
        if leaf in ("norm1", "norm2") or name == "final.norm":
            z = 0.2 * z
        elif leaf in ("norm", "out"):
            z = 1 + 0.2 * z
        elif leaf == "sink":
            z = 1 + z
        elif leaf == "rel":
            z = 1.5 * z
        elif leaf == "A_log":
            z = 0.7 * z - 0.5
        elif leaf == "dt_bias":
            z = 1.5 * z - 2
        elif leaf == "conv":
            z = 0.5 * z
        elif leaf == "step":
            z = 0.5 * z
        elif leaf in ("D", "b") and len(shape) == 1:
            z = 0.7 * z
        elif leaf != "embed":
            z = z * 1.4 / math.sqrt(shape[-1])
        out[name] = z.to(torch.bfloat16).double()
    return out
