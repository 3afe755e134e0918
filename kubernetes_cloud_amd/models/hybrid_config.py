"""Configuration of per-layer mixed decoders (``models.hybrid_lm``): every layer names its own token mixer and
feed-forward, so a design is a list of layer specs plus a few model-wide constants."""
from __future__ import annotations

import dataclasses


def _up8(n: int) -> int:
    return -(-n // 8) * 8


def aligned_parts(sizes: dict) -> tuple[dict, int]:
    """Row (or column) blocks side by side, each starting at a multiple of 8: {name: (offset, size)}, total."""
    out, o = {}, 0
    for name, n in sizes.items():
        out[name] = (o, n)
        o = _up8(o + n)
    return out, o


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

    @property
    def extra(self) -> dict:
        """Parameters beside the in and out projections: name -> shape."""
        return {"lam": (4, self.dim)}


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

    @property
    def extra(self) -> dict:
        return {"b_z": (self.width,), "b_x": (self.width,)}


@dataclasses.dataclass(frozen=True)
class LatentAttentionSpec:
    """Attention whose queries come from a normed latent of size ``q_rank`` and whose keys and values come from
    a cached, normed latent of size ``kv_rank`` plus one rotated key part of size ``rot_dim`` shared by all
    heads; a learned sink joins each head's softmax."""
    heads: int
    dim: int
    vdim: int
    rot_dim: int
    q_rank: int
    kv_rank: int
    scale: float
    rot_base: float
    rot_dims: int               # of rot_dim, rotated in interleaved pairs

    def __post_init__(self):
        if self.rot_dims % 2 or not 0 <= self.rot_dims <= self.rot_dim:
            raise ValueError(f"{self.rot_dims} of {self.rot_dim} dimensions rotate in pairs")

    @property
    def parts(self) -> dict:
        return aligned_parts({"dq": self.q_rank, "dkv": self.kv_rank + self.rot_dim})[0]

    @property
    def in_rows(self) -> int:
        return aligned_parts({"dq": self.q_rank, "dkv": self.kv_rank + self.rot_dim})[1]

    @property
    def out_cols(self) -> int:
        return self.heads * self.vdim

    @property
    def extra(self) -> dict:
        H, C = self.heads, self.kv_rank
        return {"q_norm": (self.q_rank,), "kv_norm": (C,), "uq": (H * (self.dim + self.rot_dim), self.q_rank),
                "ukv": (H * (self.dim + self.vdim), C), "sink": (H,)}


@dataclasses.dataclass(frozen=True)
class GeneralDeltaSpec:
    """Generalised delta rule: a decay and a removal rate per head and key channel, unit removal keys.
    ``decay_rank``: inner size of the two-step decay projection (None: the head size)."""
    heads: int
    dim: int
    decay_rank: int | None = None

    general = True
    taps = 0

    @property
    def kv_heads(self) -> int:
        return self.heads

    @property
    def vdim(self) -> int:
        return self.dim

    @property
    def rank_w(self) -> int:
        return self.decay_rank or self.dim

    @property
    def _sizes(self) -> dict:
        n = self.heads * self.dim
        return {"r": n, "k": n, "v": n, "g": n, "a": n, "w1": self.rank_w}

    @property
    def parts(self) -> dict:
        return aligned_parts(self._sizes)[0]

    @property
    def in_rows(self) -> int:
        return aligned_parts(self._sizes)[1]

    @property
    def out_cols(self) -> int:
        return self.heads * self.dim

    @property
    def extra(self) -> dict:
        n = self.heads * self.dim
        return {"w2": (n, self.rank_w), "w0": (n,), "a_bias": (n,), "gain": (n,)}


@dataclasses.dataclass(frozen=True)
class ChannelDeltaSpec:
    """Gated delta rule with a decay per head and key channel: q / k heads shared by groups of value heads,
    short causal convolutions before unit keys and queries, two-step decay and gate projections (inner sizes
    ``decay_rank`` / ``gate_rank``, None: the value head size)."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int
    decay_rank: int | None = None
    gate_rank: int | None = None

    general = False

    def __post_init__(self):
        if self.heads % self.kv_heads:
            raise ValueError(f"{self.heads} heads over {self.kv_heads} query/key heads")

    @property
    def rank_w(self) -> int:
        return self.decay_rank or self.vdim

    @property
    def rank_g(self) -> int:
        return self.gate_rank or self.vdim

    @property
    def conv_channels(self) -> int:
        return 2 * self.kv_heads * self.dim + self.heads * self.vdim

    @property
    def _sizes(self) -> dict:
        n = self.kv_heads * self.dim
        return {"q": n, "k": n, "v": self.heads * self.vdim, "a1": self.rank_w, "g1": self.rank_g, "b": self.heads}

    @property
    def parts(self) -> dict:
        return aligned_parts(self._sizes)[0]

    @property
    def in_rows(self) -> int:
        return aligned_parts(self._sizes)[1]

    @property
    def out_cols(self) -> int:
        return self.heads * self.vdim

    @property
    def extra(self) -> dict:
        H = self.heads
        return {"conv": (self.conv_channels, self.taps), "a2": (H * self.dim, self.rank_w), "dt_bias": (H * self.dim,),
                "a_log": (H,), "g2": (H * self.vdim, self.rank_g), "gain": (self.vdim,)}


@dataclasses.dataclass(frozen=True)
class BiasedAttentionSpec:
    """Attention without rotation: RMS-normed queries and keys, a learned bias by bucketed distance (``bias_rows``
    buckets, spaced in ln(distance) up to ``bias_max`` beyond the near half), a learned sink per head, and a
    sigmoid gate on the heads' outputs."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    bias_max: float
    bias_rows: int = 32

    def __post_init__(self):
        if self.heads % self.kv_heads:
            raise ValueError(f"{self.heads} query heads over {self.kv_heads} key/value heads")

    @property
    def _sizes(self) -> dict:
        return {"q": self.heads * self.dim, "k": self.kv_heads * self.dim, "v": self.kv_heads * self.vdim,
                "g": self.heads * self.vdim}

    @property
    def parts(self) -> dict:
        return aligned_parts(self._sizes)[0]

    @property
    def in_rows(self) -> int:
        return aligned_parts(self._sizes)[1]

    @property
    def out_cols(self) -> int:
        return self.heads * self.vdim

    @property
    def extra(self) -> dict:
        return {"q_norm": (self.dim,), "k_norm": (self.dim,), "rel": (self.bias_rows, self.heads), "sink": (self.heads,)}


@dataclasses.dataclass(frozen=True)
class HeadDeltaSpec:
    """Gated delta rule with one decay per head: q / k heads shared by groups of value heads, short causal
    convolutions before unit keys and queries, a silu gate on the normed read-out."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int

    def __post_init__(self):
        if self.heads % self.kv_heads:
            raise ValueError(f"{self.heads} heads over {self.kv_heads} query/key heads")

    @property
    def conv_channels(self) -> int:
        return 2 * self.kv_heads * self.dim + self.heads * self.vdim

    @property
    def _sizes(self) -> dict:
        n = self.kv_heads * self.dim
        return {"q": n, "k": n, "v": self.heads * self.vdim, "g": self.heads * self.vdim, "b": self.heads, "a": self.heads}

    @property
    def parts(self) -> dict:
        return aligned_parts(self._sizes)[0]

    @property
    def in_rows(self) -> int:
        return aligned_parts(self._sizes)[1]

    @property
    def out_cols(self) -> int:
        return self.heads * self.vdim

    @property
    def extra(self) -> dict:
        H = self.heads
        return {"conv": (self.conv_channels, self.taps), "dt_bias": (H,), "a_log": (H,), "gain": (self.vdim,)}


@dataclasses.dataclass(frozen=True)
class SsdSpec:
    """Selective state space with one decay per head (state-space duality): ``groups`` of heads share B and C of
    size ``state``; a short causal convolution with a bias; the gated output is normed in ``norm_groups`` parts."""
    heads: int
    groups: int
    state: int
    vdim: int
    taps: int
    norm_groups: int = 1

    def __post_init__(self):
        if self.heads % self.groups:
            raise ValueError(f"{self.heads} heads over {self.groups} groups")
        if self.heads * self.vdim % self.norm_groups:
            raise ValueError(f"{self.heads * self.vdim} channels in {self.norm_groups} equal parts")

    @property
    def conv_channels(self) -> int:
        return 2 * self.groups * self.state + self.heads * self.vdim

    @property
    def _sizes(self) -> dict:
        n = self.groups * self.state
        return {"C": n, "B": n, "x": self.heads * self.vdim, "z": self.heads * self.vdim, "dt": self.heads}

    @property
    def parts(self) -> dict:
        return aligned_parts(self._sizes)[0]

    @property
    def in_rows(self) -> int:
        return aligned_parts(self._sizes)[1]

    @property
    def out_cols(self) -> int:
        return self.heads * self.vdim

    @property
    def extra(self) -> dict:
        """``conv`` / ``conv_b``: channels in the order C, B, x."""
        H = self.heads
        return {"conv": (self.conv_channels, self.taps), "conv_b": (self.conv_channels,), "dt_bias": (H,), "a_log": (H,),
                "skip": (H,), "gain": (self.out_cols,)}


@dataclasses.dataclass(frozen=True)
class SideBySideSpec:
    """Two mixers of the same input, each with an output projection and an output norm of its own; the layer adds
    ``mul`` times the sum of the normed outputs."""
    left: BiasedAttentionSpec | HeadDeltaSpec | SsdSpec
    right: BiasedAttentionSpec | HeadDeltaSpec | SsdSpec
    mul: float = 0.5

    @property
    def in_rows(self) -> int:
        return self.left.in_rows + self.right.in_rows

    @property
    def out_cols(self) -> int:
        return self.left.out_cols + self.right.out_cols

    @property
    def extra(self) -> dict:
        return {f"{s}.{k}": v for s in ("left", "right") for k, v in getattr(self, s).extra.items()}


@dataclasses.dataclass(frozen=True)
class PooledAttentionSpec:
    """Rotated sliding-window attention that sees the whole blocks of ``pool`` tokens before its ``window`` as their
    means: biased projections, queries and keys RMS-normed over all heads at once, a learned sink per head.
    ``rot_scaling``: (factor, low, high, original) of the three-band frequency scaling, or None."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int
    pool: int
    rot_base: float
    rot_dims: int               # leading dims of a head that rotate, in pairs half of them apart
    rot_scaling: tuple | None = None

    def __post_init__(self):
        if self.heads % self.kv_heads:
            raise ValueError(f"{self.heads} query heads over {self.kv_heads} key/value heads")
        if self.rot_dims % 2 or not 0 <= self.rot_dims <= self.dim:
            raise ValueError(f"{self.rot_dims} of {self.dim} dimensions rotate in pairs")
        if self.window < 1 or self.pool < 1:
            raise ValueError(f"a window of {self.window} tokens, blocks of {self.pool}")

    @property
    def _sizes(self) -> dict:
        return {"q": self.heads * self.dim, "k": self.kv_heads * self.dim, "v": self.kv_heads * self.vdim}

    @property
    def parts(self) -> dict:
        return aligned_parts(self._sizes)[0]

    @property
    def in_rows(self) -> int:
        return aligned_parts(self._sizes)[1]

    @property
    def out_cols(self) -> int:
        return self.heads * self.vdim

    @property
    def extra(self) -> dict:
        return {"q_norm": (self.heads * self.dim,), "k_norm": (self.kv_heads * self.dim,), "sink": (self.heads,)}


@dataclasses.dataclass(frozen=True)
class MatrixMemorySpec:
    """Matrix memory with exponential gates (mLSTM): soft-capped log gates, a normaliser and a running maximum beside the
    state, read-outs normed per head and gated."""
    heads: int
    dim: int
    vdim: int
    gate_cap: float

    @property
    def _sizes(self) -> dict:
        n, e = self.heads * self.dim, self.heads * self.vdim
        return {"q": n, "k": n, "v": e, "g": e, "i": self.heads, "f": self.heads}

    @property
    def parts(self) -> dict:
        return aligned_parts(self._sizes)[0]

    @property
    def in_rows(self) -> int:
        return aligned_parts(self._sizes)[1]

    @property
    def out_cols(self) -> int:
        return self.heads * self.vdim

    @property
    def extra(self) -> dict:
        return {"i_bias": (self.heads,), "f_bias": (self.heads,), "gain": (self.heads * self.vdim,)}


@dataclasses.dataclass(frozen=True)
class SumSpec:
    """Two mixers of the same input behind one input and one output projection: each side's rows are weighted, then
    both close in one product."""
    left: PooledAttentionSpec | MatrixMemorySpec
    right: PooledAttentionSpec | MatrixMemorySpec
    left_mul: float = 1.0
    right_mul: float = 1.0

    @property
    def in_rows(self) -> int:
        return self.left.in_rows + self.right.in_rows

    @property
    def out_parts(self) -> dict:
        return aligned_parts({"left": self.left.out_cols, "right": self.right.out_cols})[0]

    @property
    def out_cols(self) -> int:
        return aligned_parts({"left": self.left.out_cols, "right": self.right.out_cols})[1]

    @property
    def extra(self) -> dict:
        return {f"{s}.{k}": v for s in ("left", "right") for k, v in getattr(self, s).extra.items()}


@dataclasses.dataclass(frozen=True)
class DenseSpec:
    """W_down act(W_up h); ``act``: "gelu" (exact) or "relu2" (squared ReLU)."""
    ff: int
    act: str = "gelu"


@dataclasses.dataclass(frozen=True)
class GatedDenseSpec:
    """W_down (gelu_tanh(W_gate h + b) * (W_up h + b)) + b."""
    ff: int


@dataclasses.dataclass(frozen=True)
class MoESpec:
    """Routed gated experts. ``score`` "sigmoid": the largest scores are the weights; "softmax": the largest scores plus
    ``correction`` within the ``keep`` best of ``groups`` equal groups, weighted by the scores over their sum.
    ``identity``: router outputs behind the experts' whose choice passes the token on."""
    experts: int
    top: int
    ff: int
    shared_ff: int = 0          # always-on expert (0: none)
    scale_in: bool = True       # the router weight scales the expert's input (False: its output)
    shared_gate: bool = True    # ... behind a per-token gate
    score: str = "sigmoid"
    identity: int = 0
    groups: int = 1
    keep: int = 1
    correction: bool = False

    def __post_init__(self):
        n = self.outputs
        if n % self.groups or not 1 <= self.keep <= self.groups:
            raise ValueError(f"{self.keep} of {self.groups} groups of {n} router outputs")
        if not 1 <= self.top <= n // self.groups * self.keep:
            raise ValueError(f"top {self.top} of {n // self.groups * self.keep} experts")
        if self.score == "sigmoid" and (self.identity or self.groups > 1 or self.correction):
            raise ValueError("identity experts, groups and corrections belong to softmax routers")

    @property
    def outputs(self) -> int:
        """Rows of the router."""
        return self.experts + self.identity


@dataclasses.dataclass(frozen=True)
class LayerSpec:
    mixer: (DiffAttentionSpec | GatedRecurrenceSpec | LatentAttentionSpec | GeneralDeltaSpec | ChannelDeltaSpec |
            BiasedAttentionSpec | HeadDeltaSpec | SsdSpec | SideBySideSpec | PooledAttentionSpec | MatrixMemorySpec | SumSpec)
    mlp: DenseSpec | GatedDenseSpec | MoESpec | None


@dataclasses.dataclass(frozen=True)
class LoopSpec:
    """Layers ``start`` .. ``stop - 1`` run ``times`` times in a row with the same weights; every pass has its
    own cache or state. ``entry``: a pass starts from a projection of the stream beside the embedding output, plus
    one vector per pass."""
    start: int
    stop: int
    times: int
    entry: bool = False


@dataclasses.dataclass
class HybridConfig:
    arch: str
    vocab_size: int
    hidden: int
    layers: tuple
    norm_eps: float = 1e-5
    residual_mult: float = 1.0
    # one norm feeds mixer and feed-forward | "sandwich": in turn, normed before and after | "prenorm": in turn,
    # RMS-normed before, gains stored around zero | "postnorm": in turn, RMS-normed after, gains of one number
    block: str = "parallel"
    embed_scale: float = 1.0
    logit_scale: float = 1.0
    tied: bool = False           # the embedding table is the output projection
    logit_softcap: float = 0.0   # cap tanh(logits / cap); 0: none
    loop: LoopSpec | None = None
    max_pos: int = 8192          # serving default; the design itself sets no limit
    bos_token_id: int | None = None
    eos_token_id: int | None = None
    pad_token_id: int | None = None
    hf: dict = dataclasses.field(default_factory=dict, repr=False)

    @property
    def n_layers(self) -> int:
        return len(self.layers)

    @property
    def runs(self) -> tuple:
        """Layer indices in the order they run."""
        n, lp = len(self.layers), self.loop
        if lp is None:
            return tuple(range(n))
        if not 0 <= lp.start <= lp.stop <= n or lp.times < 0:
            raise ValueError(f"loop {lp} over {n} layers")
        return (*range(lp.start), *(tuple(range(lp.start, lp.stop)) * lp.times), *range(lp.stop, n))

    @property
    def opens(self) -> tuple:
        """For every run, the loop pass it opens, or None."""
        lp = self.loop
        if lp is None or lp.start == lp.stop:
            return (None,) * len(self.runs)
        n = lp.stop - lp.start
        return tuple((r - lp.start) // n if 0 <= r - lp.start < n * lp.times and (r - lp.start) % n == 0 else None
                     for r in range(len(self.runs)))

    def to_hf(self) -> dict:
        return dict(self.hf)

    def n_params(self) -> int:
        def numel(shape):
            n = 1
            for x in shape:
                n *= x
            return n

        d, pre, post = self.hidden, self.block == "prenorm", self.block == "postnorm"
        scalar = self.block in ("parallel", "postnorm")  # norms with one number
        n = (1 if self.tied else 2) * self.vocab_size * d + (1 if scalar else d)
        if self.loop is not None and self.loop.entry:
            n += (2 * d + self.loop.times) * d
        for L in self.layers:
            n += (L.mixer.in_rows + L.mixer.out_cols) * d + sum(numel(s) for s in L.mixer.extra.values())
            n += 2 * d if isinstance(L.mixer, SideBySideSpec) else 0
            n += 1 + L.mixer.in_rows if post else 1 + d if scalar else d if pre else 3 * d
            if isinstance(L.mlp, DenseSpec):
                n += 2 * d * L.mlp.ff + (d if pre else 0)
            elif isinstance(L.mlp, GatedDenseSpec):
                n += 3 * d * L.mlp.ff + 2 * L.mlp.ff + 4 * d
            elif L.mlp is not None:
                m = L.mlp
                n += d * (m.outputs + 3 * m.experts * m.ff + 3 * m.shared_ff) + (m.outputs if m.correction else 0)
                n += d if m.shared_ff and m.shared_gate else 0
                n += 1 if post else 0
        return n


__all__ = ["HybridConfig", "LayerSpec", "LoopSpec", "DiffAttentionSpec", "GatedRecurrenceSpec", "LatentAttentionSpec",
           "GeneralDeltaSpec", "ChannelDeltaSpec", "BiasedAttentionSpec", "HeadDeltaSpec", "SsdSpec", "SideBySideSpec",
           "PooledAttentionSpec", "MatrixMemorySpec", "SumSpec",
           "DenseSpec", "GatedDenseSpec", "MoESpec", "aligned_parts"]
