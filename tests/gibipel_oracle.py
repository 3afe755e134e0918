"""Plain, slow Gibipel forward used as the oracle of the Gibipel tests: whole sequences, one function per mechanism, a
loop over tokens and heads wherever that is the definition, float64. It shares no code with the product path.

``weights`` is a dict of float64 tensors under the checkpoint's tensor names, ``cfg`` the parsed config.json.
"""
import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def log_sigmoid(z):
    return torch.clamp(z, max=0) - torch.log1p(torch.exp(-z.abs()))


def frequencies(rot):
    """Radians per position of each rotated pair; slow ones are stretched (three bands by wavelength)."""
    out = []
    s = rot.get("scaling")
    for i in range(rot["dims"] // 2):
        f = rot["base"] ** (-2 * i / rot["dims"])
        if s:
            wave = 2 * math.pi / f
            if wave > s["original"] / s["low"]:
                f = f / s["factor"]
            elif wave >= s["original"] / s["high"]:
                mix = (s["original"] / wave - s["low"]) / (s["high"] - s["low"])
                f = (1 - mix) * f / s["factor"] + mix * f
        out.append(f)
    return out


def rotate(x, rot):
    """[T, heads, D], row t at position t: pairs (i, i + dims / 2) of a head's first dims turn."""
    y, n = x.clone(), rot["dims"] // 2
    t = torch.arange(x.shape[0], dtype=x.dtype)[:, None]
    for i, f in enumerate(frequencies(rot)):
        c, s, u, v = torch.cos(t * f), torch.sin(t * f), x[:, :, i], x[:, :, i + n]
        y[:, :, i], y[:, :, i + n] = u * c - v * s, v * c + u * s
    return y


def window(i, size):
    """First token that position i sees."""
    return max(0, i - size + 1)


def blocks_seen(i, size, pool):
    """How many whole blocks end before the window of position i."""
    n = 0
    while n * pool + pool - 1 <= i - size:
        n += 1
    return n


def block_means(x, pool):
    """[T, D] -> means of the whole blocks."""
    n = x.shape[0] // pool
    return x[:n * pool].view(n, pool, x.shape[1]).mean(1)


def sink_softmax(scores, sink):
    """exp(s_j) / (exp(sink) + sum_j exp(s_j))."""
    m = max(float(scores.max()), float(sink))
    e = torch.exp(scores - m)
    return e / (e.sum() + math.exp(float(sink) - m))


def pooled_attention(q, k, v, sink, mx):
    """Rotated q [T, H, D], k [T, G, D] and v [T, G, E] -> [T, H, E]: the tokens of a sliding window and the means of
    whole blocks before it, one softmax with a sink."""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    size, pool = mx["mask"]["size"], mx["mask"]["pool"]
    kb = [block_means(k[:, g], pool) for g in range(G)]
    vb = [block_means(v[:, g], pool) for g in range(G)]
    out = torch.empty(T, H, v.shape[2], dtype=q.dtype)
    for i in range(T):
        lo, n = window(i, size), blocks_seen(i, size, pool)
        for h in range(H):
            g = h // (H // G)
            keys, values = torch.cat([kb[g][:n], k[lo:i + 1, g]]), torch.cat([vb[g][:n], v[lo:i + 1, g]])
            out[i, h] = sink_softmax((keys @ q[i, h]) * mx["scale"], sink[h]) @ values
    return out


def attention_inputs(h, w, p, mx, eps):
    """Biased projections; queries and keys normed over all heads at once, then rotated."""
    T, D = h.shape[0], mx["dim"]
    q, k, v = (h @ w[p + n].T + w[p + n + ".b"] for n in "qkv")
    q, k = rms(q, eps) * w[p + "q.norm"], rms(k, eps) * w[p + "k.norm"]
    q, k = rotate(q.view(T, mx["heads"], D), mx["rot"]), rotate(k.view(T, mx["kv_heads"], D), mx["rot"])
    return q, k, v.view(T, mx["kv_heads"], mx["vdim"])


def attention(h, w, p, mx, eps):
    q, k, v = attention_inputs(h, w, p, mx, eps)
    return pooled_attention(q, k, v, w[p + "sink"], mx).reshape(h.shape[0], -1) @ w[p + "o"].T


def memory_reads(q, k, v, i, f):
    """One head: q, k [T, D], v [T, E], log gates i, f [T] -> read-outs [T, E] of a matrix memory and its normaliser,
    both kept relative to a running maximum."""
    T, D, E = q.shape[0], q.shape[1], v.shape[1]
    S, n, m = torch.zeros(D, E, dtype=q.dtype), torch.zeros(D, dtype=q.dtype), 0.0
    out = torch.empty(T, E, dtype=q.dtype)
    for t in range(T):
        top = max(float(f[t]) + m, float(i[t]))
        keep, put = math.exp(float(f[t]) + m - top), math.exp(float(i[t]) - top)
        S = keep * S + put * torch.outer(k[t], v[t])
        n = keep * n + put * k[t]
        m = top
        out[t] = (S.T @ q[t]) / (max(abs(float(n @ q[t])), math.exp(-m)) + 1e-6)
    return out


def memory_gates(h, w, p, mx):
    """Log input and forget gates [T, H], soft-capped before the sigmoid."""
    cap = mx["gate_cap"]
    i = cap * torch.tanh((h @ w[p + "i"].T + w[p + "i.b"]) / cap)
    f = log_sigmoid(cap * torch.tanh((h @ w[p + "f"].T + w[p + "f.b"]) / cap))
    return i, f


def memory(h, w, p, mx, eps):
    H, D, E = mx["heads"], mx["dim"], mx["vdim"]
    T = h.shape[0]
    q, k = (h @ w[p + "q"].T).view(T, H, D) * D ** -0.5, (h @ w[p + "k"].T).view(T, H, D)
    v = (h @ w[p + "v"].T).view(T, H, E)
    i, f = memory_gates(h, w, p, mx)
    o = torch.stack([memory_reads(q[:, a], k[:, a], v[:, a], i[:, a], f[:, a]) for a in range(H)], 1)
    o = rms(o, eps).reshape(T, H * E) * w[p + "norm"]
    return (o * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def side_by_side(h, w, p, mx, eps):
    return mx["left_scale"] * attention(h, w, p + "left.", mx["left"], eps) + \
        mx["right_scale"] * memory(h, w, p + "right.", mx["right"], eps)


def gated(h, w, p):
    return (silu(h @ w[p + ".gate"].T) * (h @ w[p + ".up"].T)) @ w[p + ".down"].T


def choose(scores, correction, groups, top):
    """One token's experts: the largest corrected scores within the groups whose best one is largest."""
    c = [float(s) + float(b) for s, b in zip(scores, correction)]
    size = len(c) // groups["count"]
    best = sorted(range(groups["count"]), key=lambda g: -max(c[g * size:(g + 1) * size]))[:groups["keep"]]
    left = [e for e in range(len(c)) if e // size in best]
    return sorted(left, key=lambda e: -c[e])[:top]


def routed(h, w, p, mlp):
    r = mlp["router"]
    s = torch.softmax(h @ w[p + "router"].T, -1)
    fix = w.get(p + "correction")
    fix = torch.zeros(s.shape[1], dtype=s.dtype) if fix is None else fix
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        ids = choose(s[t], fix, r.get("groups") or {"count": 1, "keep": 1}, r["top"])
        total = sum(float(s[t, e]) for e in ids) + 1e-20
        for e in ids:
            y = gated(h[t:t + 1], w, f"{p}e{e}")[0] if e < r["experts"] else h[t]
            out[t] += float(s[t, e]) / total * y
    return out + gated(h, w, p + "shared") if mlp.get("shared") else out


def forward(cfg, w, tokens, layers_out=None):
    """Logits [T, vocab]; ``layers_out`` collects the stream after every layer."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][tokens] * cfg["embedding"]["scale"]
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = x + rms(side_by_side(x, w, p + "mix.", L["mixer"], eps), eps) * w[p + "norm1"]
        if L.get("mlp"):
            x = x + rms(routed(x, w, p + "mlp.", L["mlp"]), eps) * w[p + "norm2"]
        if layers_out is not None:
            layers_out.append(x)
    return (rms(x, eps) * w["final.norm"]) @ w["head"].T * cfg["logit_scale"]


def shapes(cfg):
    """Tensor name -> shape."""
    d, V = cfg["width"], cfg["vocab"]
    out = {"embed": (V, d), "head": (V, d), "final.norm": ()}
    for i, L in enumerate(cfg["layers"]):
        p, a, b = f"l{i}.", L["mixer"]["left"], L["mixer"]["right"]
        m, H, D, E = p + "mix.left.", a["heads"], a["dim"], a["vdim"]
        nq, nk, nv = H * D, a["kv_heads"] * D, a["kv_heads"] * E
        for n, c in (("q", nq), ("k", nk), ("v", nv)):
            out.update({m + n: (c, d), m + n + ".b": (c,)})
        out.update({p + "norm1": (), m + "q.norm": (nq,), m + "k.norm": (nk,), m + "sink": (H,), m + "o": (d, H * E)})
        m, H, D, E = p + "mix.right.", b["heads"], b["dim"], b["vdim"]
        out.update({m + "q": (H * D, d), m + "k": (H * D, d), m + "v": (H * E, d), m + "g": (H * E, d), m + "o": (d, H * E),
                    m + "norm": (H * E,), **{m + n: (H, d) for n in "if"}, **{m + n + ".b": (H,) for n in "if"}})
        if L.get("mlp"):
            r, m = L["mlp"]["router"], p + "mlp."
            E = r["experts"] + r.get("identity", 0)
            out.update({p + "norm2": (), m + "router": (E, d), m + "correction": (E,)})
            ffs = {f"e{e}": L["mlp"]["expert"]["ff"] for e in range(r["experts"])}
            if L["mlp"].get("shared"):
                ffs["shared"] = L["mlp"]["shared"]["ff"]
            for n, F in ffs.items():
                out.update({f"{m}{n}.gate": (F, d), f"{m}{n}.up": (F, d), f"{m}{n}.down": (d, F)})
    return out


def random_weights(cfg, seed=0):
    """Weights whose mechanisms all matter: query rows that pick keys out, gates on both sides of their caps,
    corrections that change the choice. bfloat16 values in float64."""
    g = torch.Generator().manual_seed(seed)
    r = lambda *s: torch.randn(s, generator=g)  # noqa: E731
    w = {}
    for n, s in shapes(cfg).items():
        last = n.rsplit(".", 1)[-1]
        if n.endswith(("norm1", "norm2", "final.norm")):
            t = 0.6 + 0.2 * r(*s)
        elif last == "norm":
            t = 1 + 0.3 * r(*s)
        elif last == "sink":
            t = 1 + r(*s)
        elif last == "correction":
            t = 0.15 * r(*s)
        elif n.endswith("f.b"):
            t = 2 + 2 * r(*s)
        elif last == "b":
            t = 0.5 * r(*s)
        elif n == "embed":
            t = r(*s)
        elif last in ("i", "f"):
            t = r(*s) * 1.5 * s[1] ** -0.5
        else:
            t = r(*s) * s[-1] ** -0.5
        w[n] = t.to(torch.bfloat16).double()
    return w
