"""Configuration of per-layer mixed decoders (``models.hybrid_lm``): every layer names its own token mixer and
feed-forward, so a design is a list of layer specs plus a few model-wide constants."""
from __future__ import annotations

import dataclasses


@dataclasses.dataclass(frozen=True)
class DiffAttentionSpec:
    """Differential attention: two softmax maps of size ``dim`` per head over shared values of size ``vdim``."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    diff: float                 # offset of lambda; the output keeps 1 - diff
    temp_coef: float = 0.0      # query temperature 1 + coef ln(floor((pos + 1) / every) + 1)
    temp_every: float = 0.0     # 0: none

    def __post_init__(self):
        if self.heads % self.kv_heads:
            raise ValueError(f"{self.heads} query heads over {self.kv_heads} key/value heads")

    @property
    def in_rows(self) -> int:
        return 2 * (self.heads + self.kv_heads) * self.dim + self.kv_heads * self.vdim

    @property
    def out_cols(self) -> int:
        return self.heads * self.vdim


@dataclasses.dataclass(frozen=True)
class GatedRecurrenceSpec:
    """minGRU: an element-wise gated recurrence of ``width`` channels with an output gate."""
    width: int

    @property
    def in_rows(self) -> int:
        return 3 * self.width

    @property
    def out_cols(self) -> int:
        return self.width


@dataclasses.dataclass(frozen=True)
class DenseSpec:
    ff: int


@dataclasses.dataclass(frozen=True)
class MoESpec:
    experts: int
    top: int
    ff: int
    shared_ff: int = 0          # always-on expert behind a per-token gate (0: none)
    scale_in: bool = True       # the router weight scales the expert's input (False: its output)

    def __post_init__(self):
        if not 1 <= self.top <= self.experts:
            raise ValueError(f"top {self.top} of {self.experts} experts")


@dataclasses.dataclass(frozen=True)
class LayerSpec:
    mixer: DiffAttentionSpec | GatedRecurrenceSpec
    mlp: DenseSpec | MoESpec | None


@dataclasses.dataclass
class HybridConfig:
    arch: str
    vocab_size: int
    hidden: int
    layers: tuple
    norm_eps: float = 1e-5
    residual_mult: float = 1.0
    max_pos: int = 8192          # serving default; the design itself sets no limit
    bos_token_id: int | None = None
    eos_token_id: int | None = None
    pad_token_id: int | None = None
    hf: dict = dataclasses.field(default_factory=dict, repr=False)

    @property
    def n_layers(self) -> int:
        return len(self.layers)

    def to_hf(self) -> dict:
        return dict(self.hf)

    def n_params(self) -> int:
        d, n = self.hidden, 2 * self.vocab_size * self.hidden + 1
        for L in self.layers:
            n += 1 + d + (L.mixer.in_rows + L.mixer.out_cols) * d
            n += 4 * L.mixer.dim if isinstance(L.mixer, DiffAttentionSpec) else 2 * L.mixer.width
            if isinstance(L.mlp, DenseSpec):
                n += 2 * d * L.mlp.ff
            elif L.mlp is not None:
                n += d * (L.mlp.experts + 3 * L.mlp.experts * L.mlp.ff)
                n += d * (3 * L.mlp.shared_ff + 1) if L.mlp.shared_ff else 0
        return n


__all__ = ["HybridConfig", "LayerSpec", "DiffAttentionSpec", "GatedRecurrenceSpec", "DenseSpec", "MoESpec"]
