"""Plain, slow Rezusun forward used as the oracle of the Rezusun tests: whole sequences, one function per
mechanism, a loop over tokens wherever a recurrence is the definition, float64. It shares no code with the
product path.

``weights`` is a dict of float64 tensors under the checkpoint's tensor names, ``cfg`` the parsed config.json.
"""
import math

import torch


def layer_norm(x, gain, eps):
    """(x - mean) / sqrt(mean of squared deviations + eps) * gain."""
    c = x - x.mean(-1, keepdim=True)
    return c / torch.sqrt((c * c).mean(-1, keepdim=True) + eps) * gain


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def unit(x):
    """Unit vectors, with 1e-6 under the root."""
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.log1p(torch.exp(-z.abs())) + torch.clamp(z, min=0)


def rotate(x, pos, base):
    """Interleaved rotary pairs over the whole last axis of x [.., n]: (u, v) -> (u cos - v sin, v cos + u sin)."""
    n = x.shape[-1]
    out = torch.empty_like(x)
    for i in range(n // 2):
        a = pos * base ** (-2 * i / n)
        c, s = math.cos(a), math.sin(a)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i], out[..., 2 * i + 1] = u * c - v * s, v * c + u * s
    return out


def sink_softmax_row(scores, sink):
    """exp(s_j) / (exp(sink) + sum_j exp(s_j))."""
    m = max(float(scores.max()), float(sink))
    e = torch.exp(scores - m)
    return e / (e.sum() + math.exp(float(sink) - m))


def latent_attention(h, w, p, mx, eps):
    """Queries and keys/values through normed latents; every head's keys and values come from one latent c plus
    one rotated key part shared by all heads; the softmax has a sink."""
    H, D, E, R, C = mx["heads"], mx["dim"], mx["vdim"], mx["rot_dim"], mx["kv_rank"]
    T = h.shape[0]
    cq = rms(h @ w[p + "dq"].T, eps) * w[p + "dq.norm"]
    q = (cq @ w[p + "uq"].T).view(T, H, D + R)
    kv = h @ w[p + "dkv"].T
    c = rms(kv[:, :C], eps) * w[p + "dkv.norm"]
    k = (c @ w[p + "uk"].T).view(T, H, D)
    v = (c @ w[p + "uv"].T).view(T, H, E)
    nr, base = mx["rot"]["dims"], mx["rot"]["base"]
    qr, kr = q[..., D:].clone(), kv[:, C:].clone()
    for t in range(T):
        qr[t, :, :nr] = rotate(qr[t, :, :nr], t, base)
        kr[t, :nr] = rotate(kr[t, :nr], t, base)
    out = torch.empty(T, H, E, dtype=h.dtype)
    for t in range(T):
        for a in range(H):
            s = (k[:t + 1, a] @ q[t, a, :D] + kr[:t + 1] @ qr[t, a]) * mx["scale"]
            out[t, a] = sink_softmax_row(s, w[p + "sink"][a]) @ v[:t + 1, a]
    return out.reshape(T, H * E) @ w[p + "o"].T


def general_delta(h, w, p, mx, eps):
    """S <- diag(w) S - (a u) (u^T S) + k v^T per head (u the unit key), read with r after the write."""
    H, D = mx["heads"], mx["dim"]
    T = h.shape[0]
    r, k, v = ((h @ w[p + n].T).view(T, H, D) for n in ("r", "k", "v"))
    dec = torch.exp(-math.exp(-0.5) * torch.sigmoid(torch.tanh(h @ w[p + "w1"].T) @ w[p + "w2"].T + w[p + "w0"])).view(T, H, D)
    a = torch.sigmoid(h @ w[p + "a"].T + w[p + "a.b"]).view(T, H, D)
    u = unit(k)
    o = torch.empty(T, H, D, dtype=h.dtype)
    for i in range(H):
        S = torch.zeros(D, D, dtype=h.dtype)
        for t in range(T):
            S = dec[t, i][:, None] * S - torch.outer(a[t, i] * u[t, i], u[t, i] @ S) + torch.outer(k[t, i], v[t, i])
            o[t, i] = r[t, i] @ S
    y = rms(o, eps).reshape(T, H * D) * w[p + "norm"]
    return (y * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def causal_conv(x, taps):
    """Per-channel convolution over time, the last tap on the current row, zeros before the start."""
    T, n = x.shape[0], taps.shape[1]
    out = torch.zeros_like(x)
    for t in range(T):
        for i in range(n):
            if t - i >= 0:
                out[t] += taps[:, n - 1 - i] * x[t - i]
    return out


def channel_delta(h, w, p, mx, eps):
    """S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q, with a decay per head and key channel."""
    H, G, D, E = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    T = h.shape[0]
    q, k, v = (silu(causal_conv(h @ w[p + n].T, w[p + n + ".conv"])) for n in ("q", "k", "v"))
    q = unit(q.view(T, G, D)) / math.sqrt(D)
    k = unit(k.view(T, G, D))
    v = v.view(T, H, E)
    beta = torch.sigmoid(h @ w[p + "b"].T)
    dt = softplus((h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "dt_bias"]).view(T, H, D)
    g = torch.exp(-torch.exp(w[p + "A_log"])[:, None] * dt)
    o = torch.empty(T, H, E, dtype=h.dtype)
    for i in range(H):
        S, j = torch.zeros(D, E, dtype=h.dtype), i // (H // G)
        for t in range(T):
            S = g[t, i][:, None] * S
            S = S + torch.outer(k[t, j], beta[t, i] * (v[t, i] - k[t, j] @ S))
            o[t, i] = q[t, j] @ S
    gate = torch.sigmoid((h @ w[p + "g1"].T) @ w[p + "g2"].T).view(T, H, E)
    return (rms(o, eps) * w[p + "norm"] * gate).reshape(T, H * E) @ w[p + "o"].T


MIXERS = {"latent_attention": latent_attention, "general_delta": general_delta, "channel_delta": channel_delta}


def feed_forward(h, w, p):
    z = gelu_tanh(h @ w[p + "gate"].T + w[p + "gate.b"]) * (h @ w[p + "up"].T + w[p + "up.b"])
    return z @ w[p + "down"].T + w[p + "down.b"]


def order(cfg):
    """Layer indices as they run: the looped range several times in a row."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return list(range(n))
    a, b = lp["start"], lp["stop"]
    return list(range(a)) + list(range(a, b)) * lp["times"] + list(range(b, n))


def forward(cfg, weights, tokens, layers_out=None):
    """Logits [T, vocab] of one whole sequence. ``layers_out`` collects the residual stream after every run."""
    w, eps = weights, cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens)]
    for i in order(cfg):
        L, s = cfg["layers"][i], f"l{i}."
        y = MIXERS[L["type"]](layer_norm(x, w[s + "norm1"], eps), w, s + "mix.", L["mixer"], eps)
        x = x + w[s + "ls1"] * layer_norm(y, w[s + "norm1b"], eps)
        if L["mlp"] is not None:
            y = feed_forward(layer_norm(x, w[s + "norm2"], eps), w, s + "mlp.")
            x = x + w[s + "ls2"] * layer_norm(y, w[s + "norm2b"], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return layer_norm(x, w["final.norm"], eps) @ w["head"].T


def tensor_shapes(cfg, ranks):
    """Checkpoint names -> shapes; ``ranks``: {layer: {"w1" | "a1" | "g1": inner size of a two-step projection}}."""
    d, V, out = cfg["width"], cfg["vocab"], {}
    out.update({"embed": (V, d), "head": (V, d), "final.norm": (d,)})
    for i, L in enumerate(cfg["layers"]):
        s, mx = f"l{i}.", L["mixer"]
        m = s + "mix."
        out.update({s + "norm1": (d,), s + "norm1b": (d,), s + "ls1": (d,)})
        if L["type"] == "latent_attention":
            H, D, E, R, C, Q = (mx[k] for k in ("heads", "dim", "vdim", "rot_dim", "kv_rank", "q_rank"))
            out.update({m + "dq": (Q, d), m + "dq.norm": (Q,), m + "uq": (H * (D + R), Q), m + "dkv": (C + R, d),
                        m + "dkv.norm": (C,), m + "uk": (H * D, C), m + "uv": (H * E, C), m + "sink": (H,),
                        m + "o": (d, H * E)})
        elif L["type"] == "general_delta":
            n = mx["heads"] * mx["dim"]
            out.update({m + k: (n, d) for k in ("r", "k", "v", "g", "a")})
            r = ranks[i]["w1"]
            out.update({m + "a.b": (n,), m + "w1": (r, d), m + "w2": (n, r), m + "w0": (n,), m + "norm": (n,), m + "o": (d, n)})
        else:
            H, G, D, E, n = (mx[k] for k in ("heads", "kv_heads", "dim", "vdim", "conv"))
            ra, rg = ranks[i]["a1"], ranks[i]["g1"]
            for k, c in (("q", G * D), ("k", G * D), ("v", H * E)):
                out.update({m + k: (c, d), m + k + ".conv": (c, n)})
            out.update({m + "b": (H, d), m + "A_log": (H,), m + "norm": (E,), m + "a1": (ra, d), m + "a2": (H * D, ra),
                        m + "dt_bias": (H * D,), m + "g1": (rg, d), m + "g2": (H * E, rg), m + "o": (d, H * E)})
        if L["mlp"] is not None:
            f = L["mlp"]["ff"]
            q = s + "mlp."
            out.update({s + "norm2": (d,), s + "norm2b": (d,), s + "ls2": (d,), q + "gate": (f, d), q + "gate.b": (f,),
                        q + "up": (f, d), q + "up.b": (f,), q + "down": (d, f), q + "down.b": (d,)})
    return out


def random_weights(cfg, ranks, seed=0):
    """Random float64 weights that bf16 holds exactly; gains near one, decays from slow to fast, visible sinks."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg, ranks).items():
        z = torch.randn(*shape, generator=g)
        leaf = name.rsplit(".", 1)[-1]
        if "norm" in leaf:
            z = 1 + 0.2 * z
        elif leaf in ("ls1", "ls2"):
            z = 0.6 + 0.2 * z
        elif leaf == "sink":
            z = 1 + z
        elif leaf == "A_log":
            z = 0.7 * z - 0.5
        elif leaf in ("dt_bias", "w0"):
            z = 1.5 * z - 2
        elif leaf == "conv":
            z = 0.5 * z
        elif leaf in ("b",) and len(shape) == 1:
            z = 0.5 * z
        elif leaf != "embed":
            z = z * 1.4 / math.sqrt(shape[-1])
        out[name] = z.to(torch.bfloat16).double()
    return out
