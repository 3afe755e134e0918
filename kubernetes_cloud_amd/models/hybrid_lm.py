"""Decoders whose layers mix tokens differently (``HybridConfig``): differential, latent or biased attention, a gated
recurrence, a delta rule, a state space, windowed attention over block means, a matrix memory, or two of them side by
side, beside a dense, gated, routed or no feed-forward, on an fp32 residual stream.

``block`` "parallel": with h the normed stream and hs its token-shifted copy,

    x <- x + m (mixer(hs) + ff(h))

"sandwich": two sublayers in turn, each normed before and after and scaled per coordinate,

    x <- x + scale * N(mixer(N(x))),   x <- x + scale2 * N(ff(N(x)))

"prenorm": the same two sublayers, RMS-normed before only (gains stored minus one); two mixers side by side are
normed after their own output projections and averaged,

    x <- x + mixer(N(x))   |   x + mul (N(left(N(x))) + N(right(N(x)))),      x <- x + ff(N(x))

"postnorm": the same two sublayers on the stream itself, what they add RMS-normed with a gain of one number,

    x <- x + N(mixer(x)),   x <- x + N(ff(x))

The modules hold weights laid out for the kernels; the step itself (cache, state, batching) is
``engine.hybrid_runner``. Layout:

* ``w_in``   every projection of the mixer's input in one matrix ([q | k | v], [z | x | g], ...; ``spec.parts``:
  blocks start at multiples of 8 rows)
* ``w_out``  the mixer's output projection; parallel layers put the dense (or shared-expert) down projection
  beside it, [d, mixer + ff]: both branches close in one product, summed in fp32 before its rounding
* two mixers side by side: one ``w_in`` for both; ``left`` / ``right`` hold the rest of each. Summed ones share
  ``w_out`` too, [d, left | right]
* ``b_in``   biases of the input projections (zero rows where there is none)
* ``w_up``   gate and up projections of a gated feed-forward, one above the other
* experts stacked: gate-and-up [E, 2F, d], down [E, d, F]
"""
from __future__ import annotations

import torch
import torch.nn as nn

from .hybrid_config import DenseSpec, GatedDenseSpec, HybridConfig, LayerSpec, MoESpec, SideBySideSpec, SumSpec


def _p(*shape):
    return nn.Parameter(torch.empty(shape), requires_grad=False)


class SideMixer(nn.Module):
    """One of two mixers side by side: its parameters behind the layer's common input projection (``closes``: with an
    output projection and norm of its own)."""

    def __init__(self, d: int, mixer, closes: bool = True):
        super().__init__()
        self.spec = LayerSpec(mixer, None)
        for name, shape in mixer.extra.items():
            setattr(self, name, _p(*shape))
        if closes:
            self.w_out, self.out_norm = _p(d, mixer.out_cols), _p(d)


class HybridLayer(nn.Module):
    def __init__(self, cfg: HybridConfig, spec: LayerSpec):
        super().__init__()
        d, mx, mlp = cfg.hidden, spec.mixer, spec.mlp
        self.spec = spec
        self.w_in = _p(mx.in_rows, d)
        pair = isinstance(mx, SideBySideSpec)
        if pair and cfg.block != "prenorm":
            raise ValueError(f"mixers side by side belong to prenorm layers, not {cfg.block}")
        summed = isinstance(mx, SumSpec)
        if summed and cfg.block != "postnorm":
            raise ValueError(f"summed mixers belong to postnorm layers, not {cfg.block}")
        for name, shape in ({} if pair or summed else mx.extra).items():
            setattr(self, name, _p(*shape))
        if summed:
            self.left, self.right = SideMixer(d, mx.left, False), SideMixer(d, mx.right, False)
        self.moe = isinstance(mlp, MoESpec)
        if cfg.block == "postnorm":
            if mlp is not None and (not self.moe or (mlp.shared_ff and mlp.shared_gate)):
                raise ValueError("postnorm layers take routed experts, without a gate on the shared one, or no feed-forward")
            self.b_in, self.norm = _p(mx.in_rows), _p()
            self.w_out = _p(d, mx.out_cols)
            if mlp is not None:
                self.norm2, self.router = _p(), _p(mlp.outputs, d)
                self.correction = _p(mlp.outputs) if mlp.correction else None
                self.gate_up, self.down = _p(mlp.experts, 2 * mlp.ff, d), _p(mlp.experts, d, mlp.ff)
                if mlp.shared_ff:
                    self.w_up, self.w_down = _p(2 * mlp.shared_ff, d), _p(d, mlp.shared_ff)
            return
        if cfg.block == "prenorm":
            if mlp is not None and not isinstance(mlp, DenseSpec):
                raise ValueError(f"prenorm layers take a dense feed-forward or none, not {type(mlp).__name__}")
            self.norm = _p(d)
            if pair:
                self.left, self.right = SideMixer(d, mx.left), SideMixer(d, mx.right)
            else:
                self.w_out = _p(d, mx.out_cols)
            if mlp is not None:
                self.norm2, self.w_up, self.w_down = _p(d), _p(mlp.ff, d), _p(d, mlp.ff)
            return
        if cfg.block == "sandwich":
            if mlp is not None and not isinstance(mlp, GatedDenseSpec):
                raise ValueError(f"sandwich layers take a gated feed-forward or none, not {type(mlp).__name__}")
            self.norm, self.norm_b, self.scale = _p(d), _p(d), _p(d)
            self.w_out = _p(d, mx.out_cols)
            if mlp is not None:
                self.norm2, self.norm2_b, self.scale2 = _p(d), _p(d), _p(d)
                self.w_up, self.b_up = _p(2 * mlp.ff, d), _p(2 * mlp.ff)
                self.w_down, self.b_down = _p(d, mlp.ff), _p(d)
            return
        if self.moe and (mlp.score != "sigmoid" or (mlp.shared_ff and not mlp.shared_gate)):
            raise ValueError("parallel layers take sigmoid routers and a gated shared expert")
        if isinstance(mlp, GatedDenseSpec):
            raise ValueError("parallel layers take a dense or routed feed-forward, not a gated one")
        self.norm = _p()
        self.shift = _p(d)
        self.ff_cols = mlp.ff if isinstance(mlp, DenseSpec) else mlp.shared_ff if self.moe else 0
        self.w_up = _p((2 if self.moe else 1) * self.ff_cols, d) if self.ff_cols else None
        self.w_out = _p(d, mx.out_cols + self.ff_cols)
        if self.moe:
            self.router = _p(mlp.experts, d)
            self.gate_up = _p(mlp.experts, 2 * mlp.ff, d)
            self.down = _p(mlp.experts, d, mlp.ff)
            self.shared_gate = _p(1, d) if mlp.shared_ff else None

    def lam_value(self) -> float:
        """Differential attention: lambda = exp(lq1 . lk1) - exp(lq2 . lk2) + diff, one number
        for the layer (fp32); ``lam`` holds the rows lq1, lk1, lq2, lk2."""
        v = self.lam.float()
        return float(torch.exp((v[0] * v[1]).sum()) - torch.exp((v[2] * v[3]).sum())) + self.spec.mixer.diff


class HybridLM(nn.Module):
    def __init__(self, cfg: HybridConfig):
        super().__init__()
        self.cfg = cfg
        self.wte = _p(cfg.vocab_size, cfg.hidden)
        self.layers = nn.ModuleList([HybridLayer(cfg, s) for s in cfg.layers])
        self.final_norm = _p() if cfg.block in ("parallel", "postnorm") else _p(cfg.hidden)
        self.head = None if cfg.tied else _p(cfg.vocab_size, cfg.hidden)
        if cfg.loop is not None and cfg.loop.entry:
            if cfg.block != "prenorm":
                raise ValueError(f"projected loop entries belong to prenorm layers, not {cfg.block}")
            self.loop_in, self.loop_step = _p(cfg.hidden, 2 * cfg.hidden), _p(cfg.loop.times, cfg.hidden)

    @property
    def head_weight(self) -> torch.Tensor:
        return self.wte if self.head is None else self.head

    @torch.no_grad()
    def init_weights(self, std: float = 0.02, seed: int | None = None):
        g = torch.Generator(device=self.wte.device)
        if seed is not None:
            g.manual_seed(seed)
        around_zero = ("norm", "norm2", "final_norm") if self.cfg.block == "prenorm" else ()
        for name, p in self.named_parameters():
            if name.rsplit(".", 1)[-1] in around_zero:
                p.zero_()
            elif p.dim() >= 2:
                p.normal_(0.0, std, generator=g)
            elif any(k in name for k in ("norm", "scale", "gain")):
                p.fill_(1.0)
            elif name.endswith("shift"):
                p.fill_(0.5)
            else:
                p.zero_()
        return self

    def num_parameters(self) -> int:
        return sum(p.numel() for p in self.parameters())

    @torch.no_grad()
    def forward(self, input_ids: torch.Tensor) -> torch.Tensor:
        """Logits [B, S, V] of whole sequences: one step of a throw-away runner."""
        from ..engine.hybrid_runner import HybridRunner
        B, S = input_ids.shape
        r = HybridRunner(self, max_slots=B, max_len=S, use_graphs=False)
        out = r.forward_tokens([(b, row, 0, range(S)) for b, row in enumerate(input_ids.tolist())])
        return out.view(B, S, -1)


def build_hybrid(cfg: HybridConfig, device="cpu", dtype=torch.bfloat16, seed: int | None = 0) -> HybridLM:
    with torch.device("meta"):
        m = HybridLM(cfg)
    m = m.to(dtype).to_empty(device=device)
    if seed is not None:
        m.init_weights(seed=seed)
    return m


__all__ = ["HybridLM", "HybridLayer", "build_hybrid"]
