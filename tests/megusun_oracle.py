"""Plain, slow Megusun forward used as the oracle of the Megusun tests: whole sequences, one function per
mechanism, loops where a loop is the definition, float64. It shares no code with the product path.

``weights`` is a dict of float64 tensors under the checkpoint's tensor names, ``cfg`` the parsed config.json.
"""
import math

import torch


def rms_norm(x, gain, eps):
    """x / sqrt(mean(x^2) + eps) * gain, gain one number for the whole vector."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * gain


def token_shift(h, mu):
    """Row t becomes h_t + (h_(t-1) - h_t) * mu, with h_(-1) = 0."""
    out = torch.empty_like(h)
    prev = torch.zeros_like(h[0])
    for t in range(h.shape[0]):
        out[t] = h[t] + (prev - h[t]) * mu
        prev = h[t]
    return out


def query_temperature(pos, coef, every):
    return 1.0 + coef * math.log(math.floor((pos + 1) / every) + 1)


def softmax_attention_row(q, keys, values):
    """One query (already scaled) over a list of visible keys: sum_j softmax_j(q.k_j) v_j."""
    s = keys @ q
    w = torch.exp(s - s.max())
    return (w / w.sum()) @ values


def diff_lambda(w, p, diff):
    g = {n: w[p + n] for n in ("lq1", "lk1", "lq2", "lk2")}
    return float(torch.exp((g["lq1"] * g["lk1"]).sum()) - torch.exp((g["lq2"] * g["lk2"]).sum()) + diff)


def diff_attention(h, w, p, mx, eps):
    """Two softmax maps per head over shared values, combined as a1 - lambda a2, then normalised per head."""
    H, G, D, E = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    T = h.shape[0]
    q = (h @ w[p + "q"].T).view(T, H, 2, D)
    k = (h @ w[p + "k"].T).view(T, G, 2, D)
    v = (h @ w[p + "v"].T).view(T, G, E)
    lam = diff_lambda(w, p, mx["diff"])
    qt = mx.get("q_temp")
    out = torch.zeros(T, H, E, dtype=h.dtype)
    for t in range(T):
        f = mx["scale"] * (query_temperature(t, qt["coef"], qt["every"]) if qt else 1.0)
        for hd in range(H):
            g = hd // (H // G)
            a1 = softmax_attention_row(q[t, hd, 0] * f, k[:t + 1, g, 0], v[:t + 1, g])
            a2 = softmax_attention_row(q[t, hd, 1] * f, k[:t + 1, g, 1], v[:t + 1, g])
            o = a1 - lam * a2
            out[t, hd] = o / torch.sqrt((o * o).mean() + eps) * (1.0 - mx["diff"])
    return out.reshape(T, H * E) @ w[p + "o"].T


def mingru(h, w, p):
    z = torch.sigmoid(h @ w[p + "z"].T + w[p + "z.b"])
    u = h @ w[p + "x"].T + w[p + "x.b"]
    cand = torch.where(u >= 0, u + 0.5, torch.sigmoid(u))
    gate = h @ w[p + "g"].T
    s = torch.zeros_like(z[0])
    rows = []
    for t in range(h.shape[0]):
        s = (1 - z[t]) * s + z[t] * cand[t]
        rows.append(s * gate[t] * torch.sigmoid(gate[t]))
    return torch.stack(rows) @ w[p + "o"].T


def dense_ff(h, w, p):
    u = h @ w[p + "up"].T
    return (0.5 * u * (1 + torch.erf(u / math.sqrt(2.0)))) @ w[p + "down"].T


def gated_expert(x, w, p):
    g = x @ w[p + "gate"].T
    return (g * torch.sigmoid(g) * (x @ w[p + "up"].T)) @ w[p + "down"].T


def moe_route(h_row, w, p, top):
    """[(expert, weight)] of one token: the ``top`` largest sigmoid scores, the scores themselves as weights."""
    s = torch.sigmoid(w[p + "router"] @ h_row)
    order = sorted(range(len(s)), key=lambda e: -float(s[e]))[:top]
    return [(e, s[e]) for e in order]


def moe_ff(h, w, p, mlp):
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in moe_route(h[t], w, p, mlp["router"]["top"]):
            out[t] += gated_expert(s * h[t], w, p + "e%d." % e)
        if mlp.get("shared"):
            sg = torch.sigmoid(w[p + "shared.sg"] @ h[t])
            out[t] += gated_expert(h[t], w, p + "shared.") * sg
    return out


def forward(cfg, weights, tokens, want_layers=False):
    """Logits [T, vocab] of one sequence (and the residual stream after every layer)."""
    w = {k: v.double() if v.is_floating_point() else v for k, v in weights.items()}
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
    x = w["embed"][torch.tensor(tokens)]
    layers = []
    for i, L in enumerate(cfg["layers"]):
        p = "l%d." % i
        h = rms_norm(x, w[p + "norm1"], eps)
        hs = token_shift(h, w[p + "shift"])
        if L["type"] == "attention":
            y = diff_attention(hs, w, p + "mix.", L["mixer"], eps)
        else:
            y = mingru(hs, w, p + "mix.")
        if L.get("mlp"):
            if L["mlp"]["kind"] == "dense":
                y = y + dense_ff(h, w, p + "mlp.")
            else:
                y = y + moe_ff(h, w, p + "mlp.", L["mlp"])
        x = x + m * y
        layers.append(x)
    logits = rms_norm(x, w["final.norm"], eps) @ w["head"].T
    return (logits, layers) if want_layers else logits


def tensor_shapes(cfg):
    """name -> shape of every tensor of a checkpoint with this config."""
    d = cfg["width"]
    s = {"embed": (cfg["vocab"], d), "head": (cfg["vocab"], d), "final.norm": ()}
    for i, L in enumerate(cfg["layers"]):
        p, mx, mlp = "l%d." % i, L["mixer"], L.get("mlp")
        s[p + "norm1"], s[p + "shift"] = (), (d,)
        if L["type"] == "attention":
            H, G, D, E = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
            s.update({p + "mix.q": (H * 2 * D, d), p + "mix.k": (G * 2 * D, d), p + "mix.v": (G * E, d),
                      p + "mix.o": (d, H * E)})
            s.update({p + "mix." + n: (D,) for n in ("lq1", "lk1", "lq2", "lk2")})
        else:
            W = mx["width"]
            s.update({p + "mix." + n: (W, d) for n in ("z", "x", "g")})
            s.update({p + "mix.z.b": (W,), p + "mix.x.b": (W,), p + "mix.o": (d, W)})
        if not mlp:
            continue
        if mlp["kind"] == "dense":
            s.update({p + "mlp.up": (mlp["ff"], d), p + "mlp.down": (d, mlp["ff"])})
            continue
        s[p + "mlp.router"] = (mlp["router"]["experts"], d)
        for e in range(mlp["router"]["experts"]):
            f = mlp["expert"]["ff"]
            q = p + "mlp.e%d." % e
            s.update({q + "gate": (f, d), q + "up": (f, d), q + "down": (d, f)})
        if mlp.get("shared"):
            f, q = mlp["shared"]["ff"], p + "mlp.shared."
            s.update({q + "gate": (f, d), q + "up": (f, d), q + "down": (d, f), q + "sg": (1, d)})
    return s


def random_weights(cfg, seed=0, gain=1.0):
    """bfloat16 weights with activations of order one in every branch."""
    g = torch.Generator().manual_seed(seed)
    w = {}
    for name, shape in tensor_shapes(cfg).items():
        r = torch.randn(shape, generator=g)
        last = name.rsplit(".", 1)[-1]
        if last in ("norm1", "norm"):
            t = 1.0 + 0.2 * r
        elif last == "shift":
            t = 0.5 + 0.3 * r
        elif last in ("lq1", "lk1", "lq2", "lk2"):
            t = 0.2 * r
        elif last == "b":
            t = 0.5 * r
        elif name == "embed":
            t = r
        else:
            t = gain * r / math.sqrt(shape[-1])
        w[name] = t.to(torch.bfloat16)
    return w
