"""Runner of per-layer mixed decoders (``models.hybrid_lm``) on the serving engine's cache and slots.

One step function serves every batch: a flat list of tokens from several sequences, each contributing a
portion of its prompt or one decoded token.

* ``forward_tokens``  portions and decoded tokens together, each continuing its slot at any position
* ``prefill``         the engine's prompt call: the same step, without padding
* ``decode_async``    (``StepRunner``) single tokens only, captured per bucket as a HIP graph

A layer's token mixer is an object of ``mixers`` (attention over the paged cache, a recurrence over the slots'
state); around it a parallel layer takes three or four launches beside the vendor (or skinny matrix-core)
products -- residual + norm + token shift, the mixer's core, the feed-forward's activation or experts; mixer and
feed-forward close in one product -- and a sandwich layer one norm launch per sublayer (output norm, layer scale,
residual and the next norm together); a pre-norm or post-norm layer is one norm launch per sublayer too. Layers may run
several times in a row (``cfg.runs``); every run has its own cache or state.

What a sequence owns besides its KV pages lives in ``SlotState``: the last normed row of every parallel layer
(token shift) and the recurrent states. A batch with multi-token portions reads carried rows from a copy taken at
its start, because a portion's first and last rows are handled by different workgroups.
"""
from __future__ import annotations

import numpy as np
import torch
import torch.nn.functional as F

from ..ops import diff_attention as da
from ..ops import gated_scan as gs
from ..ops import moe
from ..ops import skinny_mm as smm
from ..ops.delta_rule import Portions, plan_portions
from ..ops.gemv import skinny_linear
from ..ops.latent_attention import Prompts, plan_prompts
from ..ops.norm_residual import Embedded, NormedBranch, NormedPair, NormedSum, Rows, norm_residual, postnorm, prenorm
from ..ops.rms_shift import Branch, rms_shift
from ..models.hybrid_config import MoESpec, SumSpec
from .mixers import make_mixer
from .runner import KVCache, SlotState, StepRunner

SPLIT_CLOSE = (1024, 4096)  # rows between which the closing product runs as two (HybridRunner._close)
ACTS = {2: "gelu", 3: "relu2"}  # activation codes of the streaming products
SKINNY_M = 16   # rows up to which projections stream on the skinny matrix-core kernel


class _Batch:
    """Device-side description of a step. ``single``: every entry is one token (the decode step)."""

    def __init__(self, tokens, pos, slots, max_kv):
        self.tokens, self.pos, self.slots, self.max_kv = tokens, pos, slots, max_kv
        self.T = tokens.shape[0]
        self.single = True
        self.flags = self.entry = self.tiles = self.row_of = self.portions = self.prompts = self.chunks = self.entry_slots = None
        self.multi = False
        self.row_kv = 0
        self.bufs = {}


class HybridRunner(StepRunner):
    mixed_steps = True

    def __init__(self, model, max_slots: int = 32, max_len: int | None = None, use_graphs: bool | None = None,
                 max_bans: int = 16, page_size: int | None = None, kv_pages: int | None = None):
        super().__init__(model, max_slots, max_len, use_graphs, max_bans)
        cfg, d = self.cfg, self.cfg.hidden
        if self.dtype not in (torch.bfloat16, torch.float32):
            raise TypeError(f"{cfg.arch} serves in bf16 or fp32, not {self.dtype}")
        page_size = self.default_page_size() if page_size is None else page_size
        if page_size < 16:
            raise ValueError("these layers need the paged cache (page_size >= 16)")
        if self.dtype == torch.float32 and self.device.type == "cuda":
            torch.backends.cuda.matmul.allow_tf32 = False
        self.mixers, first = [], {}  # one per layer run
        for r, i in enumerate(cfg.runs):
            self.mixers.append(make_mixer(model.layers[i], cfg, r, self._linear, first.get(i)))
            first.setdefault(i, self.mixers[-1])
        shapes, widths = [], {"shift": (len(cfg.runs), d)} if cfg.block == "parallel" else {}
        members = [m for mx in self.mixers for m in mx.members()]
        for mx in members:
            mx.index = len(shapes)
            shapes += mx.cache_shapes(page_size)
            widths.update(mx.state_widths())
        self.cache = KVCache(len(shapes), max_slots, 0, self.max_len, 0, self.device, self.dtype, page_size=page_size,
                             n_pages=kv_pages, layer_shapes=shapes)
        self.state = SlotState(max_slots, widths, self.device)
        for mx in members:
            mx.cache, mx.state = self.cache, self.state
        self._members = members
        self._forward_layers = {"parallel": self._parallel, "sandwich": self._sandwich, "prenorm": self._prenorm,
                                "postnorm": self._postnorm}[cfg.block]
        self._rules = [None if not isinstance(L.spec.mlp, MoESpec) else moe.Router(
            L.spec.mlp.score == "softmax", L.correction.float() if L.spec.mlp.correction else None, L.spec.mlp.groups,
            L.spec.mlp.keep, L.spec.mlp.identity) for L in model.layers]
        if self.device.type == "cuda":
            from ..utils import tunable
            tunable.ensure(tunable.DECODE_FILE)

    # ---------------------------------------------------------------- linear
    def _linear(self, x, w, out=None, act: int = 0, bias=None):
        """x W^T + bias (act 2: exact GELU, 3: squared ReLU). Few bf16 rows stream the weight on the GEMV / skinny matrix-core kernels."""
        T = x.shape[0]
        if (x.is_cuda and x.dtype == torch.bfloat16 and T <= SKINNY_M and w.shape[0] % 4 == 0 and smm.supported(x, w)
                and (out is None or (out.data_ptr() % 16 == 0 and out.stride(0) % 8 == 0))):
            if out is None:
                out = torch.empty(T, w.shape[0], device=x.device, dtype=x.dtype)
            if T == 1:
                return skinny_linear(x, w, bias, act, out=out)
            return smm.mm(x, w, bias, act, out=out, packed=self._packed_w(w))
        y = F.linear(x, w, bias)
        if act:
            return moe.act_rows(y, y if out is None else out, gated=False, act=ACTS[act])
        if out is not None:
            out.copy_(y)
            return out
        return y

    def _mix_and_up(self, L, h, hs, act_out):
        """Both products of the layer's norm: the mixer's projections of hs and (if the layer has one) the
        dense / shared-expert up product of h -- one launch for a few bf16 rows. -> (mix, up | None); a dense
        activation lands in ``act_out`` directly where the launch fuses it."""
        w1, w2 = L.w_in, L.w_up
        T = h.shape[0]
        dense = w2 is not None and not L.moe
        if (w2 is not None and h.is_cuda and h.dtype == torch.bfloat16 and 2 <= T <= SKINNY_M
                and w1.shape[0] % 4 == 0 and w2.shape[0] % 4 == 0 and smm.supported(hs, w1) and smm.supported(h, w2)
                and (not dense or (act_out.data_ptr() % 8 == 0 and act_out.stride(0) % 4 == 0))):
            mix = torch.empty(T, w1.shape[0], device=h.device, dtype=h.dtype)
            up = act_out if dense else torch.empty(T, w2.shape[0], device=h.device, dtype=h.dtype)
            smm.launch([smm.job([smm.part(hs, w1, packed=self._packed_w(w1))], w1.shape[0], mix),
                        smm.job([smm.part(h, w2, packed=self._packed_w(w2))], w2.shape[0], up, None,
                                2 if dense else 0)], T, h.dtype)
            return mix, (None if dense else up)
        mix = self._linear(hs, w1)
        if w2 is None:
            return mix, None
        if dense:
            self._linear(h, w2, out=act_out, act=2)
            return mix, None
        return mix, self._linear(h, w2)

    def _close(self, cat, w, cols: int):
        """The layer's closing product [mixer | ff] W_out^T. A mid-sized prompt's long K falls to a library
        kernel at half speed (2048 x 20480 x 4096: 440 us as one product, 283 us as two), so those accumulate
        the two column blocks in turn."""
        if cat.is_cuda and SPLIT_CLOSE[0] <= cat.shape[0] < SPLIT_CLOSE[1] and cat.dtype == torch.bfloat16 \
                and 0 < cols < cat.shape[1] and cols % 8 == 0 and cat.shape[1] % 8 == 0:
            return F.linear(cat[:, :cols], w[:, :cols]).addmm_(cat[:, cols:], w[:, cols:].t())
        return self._linear(cat, w)

    # ------------------------------------------------------------------ step
    def _forward(self, b: _Batch, want: torch.Tensor | None, layers_out: list | None = None) -> torch.Tensor:
        """Logits of the rows in ``want`` (None: every row). ``layers_out`` collects the residual stream after
        every layer run."""
        logits = self._linear(self._forward_layers(b, want, layers_out), self.model.head_weight)
        cap = self.cfg.logit_softcap
        return moe.act_rows(logits, logits, False, act="softcap", cap=cap) if cap else logits

    def _parallel(self, b, want, layers_out):
        """One norm and token shift a layer feed mixer and feed-forward side by side."""
        m, cfg = self.model, self.cfg
        T, d = b.T, cfg.hidden
        x, branch = None, None
        shift = self.state["shift"]
        carry = None if b.single else shift[:, b.entry_slots]
        for r, i in enumerate(cfg.runs):
            L = m.layers[i]
            src = {"embed": m.wte, "tokens": b.tokens} if r == 0 else {}
            x, h, hs = rms_shift(x, branch, cfg.residual_mult, L.norm, cfg.norm_eps, shift=L.shift,
                                 prev=shift[r] if b.single else carry[r], prev_idx=b.slots if b.single else b.entry,
                                 pos=b.pos, flags=b.flags, state=shift[r], slots=b.slots, **src)
            if layers_out is not None and r:
                layers_out.append(x.clone())
            cols = L.spec.mixer.out_cols
            cat = torch.empty(T, cols + L.ff_cols, device=h.device, dtype=h.dtype)
            mix, up = self._mix_and_up(L, h, hs, cat[:, cols:])
            self.mixers[r](mix, cat[:, :cols], b)
            y = inv = None
            if L.moe:
                mlp = L.spec.mlp
                ids, wts, sg, g = moe.route_group(h, L.router, mlp.top, L.shared_gate,
                                                  moe.tile_rows(T, mlp.top, mlp.experts, d, mlp.ff, h.dtype))
                y, inv = moe.experts(h, ids, wts, L.gate_up, L.down, g, mlp.scale_in), g.inv
                if up is not None:
                    moe.act_rows(up, cat[:, cols:], gated=True, row_scale=sg)
            branch = Branch(self._close(cat, L.w_out, cols), y, inv)
        if layers_out is not None:
            layers_out.append(rms_shift(x, branch, cfg.residual_mult, m.final_norm, cfg.norm_eps)[0])
        return rms_shift(x, branch, cfg.residual_mult, m.final_norm, cfg.norm_eps, rows=want, keep_x=False)[1]

    def _sandwich(self, b, want, layers_out):
        """Mixer and feed-forward in turn, each normed before and after and scaled per coordinate."""
        m, eps, T = self.model, self.cfg.norm_eps, b.T
        x, branch = None, None
        src = {"embed": m.wte, "tokens": b.tokens}
        for r, i in enumerate(self.cfg.runs):
            L = m.layers[i]
            x, h = norm_residual(x, branch, L.norm, eps, **src)
            if layers_out is not None and r:
                layers_out.append(x.clone())
            src = {}
            y = torch.empty(T, L.spec.mixer.out_cols, device=h.device, dtype=h.dtype)
            self.mixers[r](self._linear(h, L.w_in), y, b)
            branch = NormedBranch(self._linear(y, L.w_out), L.norm_b, L.scale)
            if L.spec.mlp is not None:
                x, h = norm_residual(x, branch, L.norm2, eps)
                y = torch.empty(T, L.spec.mlp.ff, device=h.device, dtype=h.dtype)
                moe.act_rows(self._linear(h, L.w_up), y, True, act="gelu_tanh_gated", bias=L.b_up)
                branch = NormedBranch(self._linear(y, L.w_down), L.norm2_b, L.scale2, L.b_down)
        if layers_out is not None:
            layers_out.append(norm_residual(x, branch, None, eps, **src)[0])
        return norm_residual(x, branch, m.final_norm, eps, rows=want, keep_x=False, **src)[1]

    def _prenorm(self, b, want, layers_out):
        """Mixer and feed-forward in turn, each normed before. A loop's passes start from a product of the stream
        beside the embedding output: both lie in one buffer, rounded, [x | x0]."""
        m, cfg, eps, T, d = self.model, self.cfg, self.cfg.norm_eps, b.T, self.cfg.hidden
        x, branch = Embedded(m.wte, b.tokens, cfg.embed_scale), None
        entry = cfg.loop is not None and cfg.loop.entry and cfg.loop.start < cfg.loop.stop and cfg.loop.times > 0
        xx0 = torch.empty(T, 2 * d, device=m.wte.device, dtype=m.wte.dtype) if entry else None
        for r, (i, opens) in enumerate(zip(cfg.runs, cfg.opens)):
            L = m.layers[i]
            if entry and r == 0:
                prenorm(x, None, None, eps, raw=xx0[:, d:], keep_x=False)
            if entry and opens is not None:
                out = prenorm(x, branch, None, eps, raw=xx0[:, :d], keep_x=layers_out is not None)[0]
                if layers_out is not None and r:
                    layers_out.append(out)
                x, branch = Rows(self._linear(xx0, m.loop_in), m.loop_step[opens]), None
                x, h = prenorm(x, None, L.norm, eps)
            else:
                x, h = prenorm(x, branch, L.norm, eps)
                if layers_out is not None and r:
                    layers_out.append(x.clone())
            branch = self._mix(L, self.mixers[r], h, b)
            if L.spec.mlp is not None:
                x, h = prenorm(x, branch, L.norm2, eps)
                y = self._linear(h, L.w_up, act=3 if L.spec.mlp.act == "relu2" else 2)
                branch = self._linear(y, L.w_down)
        if layers_out is not None:
            layers_out.append(prenorm(x, branch, None, eps)[0])
        return prenorm(x, branch, m.final_norm, eps, rows=want, keep_x=False)[1]

    def _postnorm(self, b, want, layers_out):
        """Mixer and feed-forward in turn on the stream itself; what they add is normed."""
        m, cfg, eps, dt = self.model, self.cfg, self.cfg.norm_eps, self.dtype
        x, branch = Embedded(m.wte, b.tokens, cfg.embed_scale), None
        for r, i in enumerate(cfg.runs):
            L = m.layers[i]
            x, h = postnorm(x, branch, eps, dt)
            if layers_out is not None and r:
                layers_out.append(x.clone())
            cols = L.spec.mixer.out_cols
            gaps = cols > L.spec.mixer.left.out_cols + L.spec.mixer.right.out_cols if isinstance(L.spec.mixer, SumSpec) else False
            y = (torch.zeros if gaps else torch.empty)(b.T, cols, device=h.device, dtype=dt)
            self.mixers[r](self._linear(h, L.w_in, bias=L.b_in), y, b)
            branch = NormedSum(L.norm, self._linear(y, L.w_out))
            if L.spec.mlp is not None:
                x, h = postnorm(x, branch, eps, dt)
                branch = self._routed(L, h, self._rules[i])
        if layers_out is not None:
            layers_out.append(postnorm(x, branch, eps, dt)[0])
        return postnorm(x, branch, eps, dt, gain=m.final_norm, mul=cfg.logit_scale, rows=want, keep_x=False)[1]

    def _routed(self, L, h, rule):
        """A post-norm layer's routed experts (and the shared one)."""
        mlp, T = L.spec.mlp, h.shape[0]
        mt = moe.tile_rows(T, mlp.top, mlp.outputs, h.shape[1], mlp.ff, h.dtype)
        ids, wts, _, g = moe.route_group(h, L.router, mlp.top, None, mt, rule)
        if mlp.shared_ff and moe.shared_ok(T, mt):
            y, a = moe.experts(h, ids, wts, L.gate_up, L.down, g, mlp.scale_in, (L.w_up, L.w_down))
            return NormedSum(L.norm2, a, y, g.inv, wts)
        y, a = moe.experts(h, ids, wts, L.gate_up, L.down, g, mlp.scale_in), None
        if mlp.shared_ff:
            act = torch.empty(T, mlp.shared_ff, device=h.device, dtype=h.dtype)
            a = self._linear(moe.act_rows(self._linear(h, L.w_up), act, gated=True), L.w_down)
        return NormedSum(L.norm2, a, y, g.inv, wts)

    def _mix(self, L, mixer, h, b):
        """A pre-norm layer's mixer -> what it adds to the stream."""
        pair = getattr(mixer, "sides", None)
        y = torch.empty(b.T, mixer.out_width if pair else L.spec.mixer.out_cols, device=h.device, dtype=h.dtype)
        mixer(self._linear(h, L.w_in), y, b)
        if not pair:
            return self._linear(y, L.w_out)
        ys, sides = [y[:, o] for o in mixer.outs], (L.left, L.right)
        d = self.cfg.hidden
        if h.is_cuda and h.dtype == torch.bfloat16 and 2 <= b.T <= SKINNY_M and d % 4 == 0 and \
                all(smm.supported(x, s.w_out) for x, s in zip(ys, sides)):  # one launch for both
            outs = [torch.empty(b.T, d, device=h.device, dtype=h.dtype) for _ in ys]
            smm.launch([smm.job([smm.part(x, s.w_out, packed=self._packed_w(s.w_out))], d, o)
                        for x, s, o in zip(ys, sides, outs)], b.T, h.dtype)
        else:
            outs = [self._linear(x, s.w_out) for x, s in zip(ys, sides)]
        return NormedPair(outs[0], L.left.out_norm, outs[1], L.right.out_norm, L.spec.mixer.mul)

    # ------------------------------------------------------- portions + tokens
    def _plan(self, entries, want_rows) -> tuple[_Batch, torch.Tensor | None]:
        """[(slot, tokens, start)] -> the batch, its host arrays uploaded in one copy."""
        ent, tok, r = [], [], 0
        for slot, toks, p0 in entries:
            ent.append((r, len(toks), p0, slot))
            tok += toks
            r += len(toks)
        T = r
        pos = np.concatenate([np.arange(p, p + n) for _, n, p, _ in ent])
        slots = np.repeat([s for _, _, _, s in ent], [n for _, n, _, _ in ent])
        single = T == len(ent)
        parts = {"tokens": np.asarray(tok, dtype=np.int64).view(np.int32), "pos": pos, "slots": slots,
                 "want": np.asarray(want_rows)}
        multi = False
        if not single:
            fl = np.zeros(T, dtype=np.int32)
            fl[[e[0] for e in ent]] |= 1
            fl[[e[0] + e[1] - 1 for e in ent]] |= 2
            parts["flags"] = fl
            parts["entry"] = np.repeat(np.arange(len(ent)), [e[1] for e in ent])
            parts["entry_slots"] = np.asarray([e[3] for e in ent])
            portions = plan_portions(ent)
            parts.update(("p_" + k, v.reshape(-1)) for k, v in portions.items())
            prompts, sizes = plan_prompts(ent)
            parts.update(("l_" + k, v.reshape(-1)) for k, v in prompts.items())
            chunks, multi = gs.plan_chunks(ent)
            parts["chunks"] = chunks.reshape(-1)
            parts["tiles"] = da.plan_tiles([e for e in ent if e[1] > 1]).reshape(-1)
            ones = [e for e in ent if e[1] == 1]
            parts["row_of"] = np.asarray([e[0] for e in ones])
        buf = torch.from_numpy(np.concatenate([p.astype(np.int32, copy=False) for p in parts.values()]))
        if self.device.type == "cuda":
            buf = buf.pin_memory().to(self.device, non_blocking=True)
        dev, o = {}, 0
        for k, p in parts.items():
            dev[k] = buf[o:o + p.size]
            o += p.size
        b = _Batch(dev["tokens"].view(torch.int64), dev["pos"], dev["slots"], int(pos.max()) + 1)
        if not single:
            b.single, b.multi = False, multi
            b.flags, b.entry, b.entry_slots = dev["flags"], dev["entry"], dev["entry_slots"].long()
            b.portions = Portions(b.pos, b.slots, **{k: dev["p_" + k].view(v.shape) for k, v in portions.items()})
            b.prompts = Prompts(**{k: dev["l_" + k].view(v.shape) for k, v in prompts.items()}, **sizes)
            b.chunks = dev["chunks"].view(-1, 6)
            b.tiles = dev["tiles"].view(-1, 4) if dev["tiles"].numel() else None
            if ones:
                b.row_of, b.row_kv = dev["row_of"], max(e[2] for e in ones) + 1
        return b, (dev["want"] if len(want_rows) else None)

    @torch.no_grad()
    def forward_tokens(self, entries, layers_out: list | None = None) -> torch.Tensor | None:
        """One batch of ``(slot, tokens, start, want)``: ``tokens`` continue the slot's sequence at position
        ``start`` (0: a new sequence takes the slot). -> logits of the wanted places (indices into
        ``tokens``) in order, [wanted, V], or None if nothing is wanted."""
        assert entries and len({e[0] for e in entries}) == len(entries), "one portion per sequence and step"
        want_rows, r = [], 0
        for slot, toks, p0, want in entries:
            if not toks:
                raise ValueError("an entry without tokens")
            if p0 + len(toks) > self.max_len:
                raise ValueError(f"sequence of {p0 + len(toks)} tokens > max_len {self.max_len}")
            if min(toks) < 0 or max(toks) >= self.V:
                raise ValueError("token id outside the vocabulary")
            want_rows += [r + w for w in want]
            r += len(toks)
            if p0 == 0:
                self.cache.release(slot)  # a reused slot starts empty
            self.cache.reserve(slot, p0 + len(toks))
        self.cache.sync()
        b, want = self._plan([e[:3] for e in entries], want_rows)
        fresh = [e[0] for e in entries if e[2] == 0]
        if fresh:
            self.seen[fresh] = 0
        self.seen[b.slots.long(), b.tokens] = 1
        if want is None:  # state and cache only: one row keeps the step's shape
            self._forward(b, b.slots.new_zeros(1), layers_out)
            return None
        return self._forward(b, want, layers_out)

    @torch.no_grad()
    def prefill(self, ids: torch.Tensor, slots: list[int], lens: list[int] | None = None,
                start: list[int] | None = None) -> torch.Tensor:
        """The engine's prompt call (``ModelRunner.prefill``): last-token logits [n, V]."""
        n, T = ids.shape
        lens = [T] * n if lens is None else [int(x) for x in lens]
        start = [0] * n if start is None else [int(x) for x in start]
        assert len(lens) == n and len(start) == n and all(0 < L <= T for L in lens)
        rows = ids.tolist()
        return self.forward_tokens([(s, row[:L], p0, [L - 1]) for s, row, L, p0 in zip(slots, rows, lens, start)])

    # ---------------------------------------------------------------- decode
    def _step_buffers(self, Bb: int, Kb: int) -> dict:
        need = {"ws": (1, torch.float32), "cnt": (1, torch.int32)}
        for mx in self._members:
            for k, (n, dt) in mx.buffers(Bb, Kb, self.dtype).items():
                need[k] = (max(n, need.get(k, (1, dt))[0]), dt)
        return {k: torch.zeros(n, device=self.device, dtype=dt) for k, (n, dt) in need.items()}

    def _step_logits(self, st, Bb, Kb):
        pk = st["pk"]
        b = _Batch(pk.d("tokens"), pk.d("pos"), pk.d("slots"), Kb)
        b.bufs = st
        return self._forward(b, None)

    def _eager_logits(self, tokens, pos, slots, kv_lens, max_kv):
        return self._forward(_Batch(tokens, pos, slots, max_kv), None)

    def _step_state(self) -> list:
        return super()._step_state() + list(self.state.t.values())

    @torch.no_grad()
    def copy_slots(self, dst: list[int], src: list[int], upto: int):
        super().copy_slots(dst, src, upto)
        if dst:
            self.state.fork(dst, src)


__all__ = ["HybridRunner"]
