"""Runner of per-layer mixed decoders (``models.hybrid_lm``) on the serving engine's cache and slots.

One step function serves every batch: a flat list of tokens from several sequences, each contributing a
portion of its prompt or one decoded token.

* ``forward_tokens``  portions and decoded tokens together, each continuing its slot at any position
* ``prefill``         the engine's prompt call: the same step, without padding
* ``decode_async``    (``StepRunner``) single tokens only, captured per bucket as a HIP graph

A layer is three or four launches around the vendor (or skinny matrix-core) products: residual + norm +
token shift, the mixer's core (attention over the paged cache, or the scan), the feed-forward's activation
or experts; mixer and feed-forward close in one product.

What a sequence owns besides its KV pages lives in ``SlotState``: the last normed row of every layer (token
shift) and the fp32 recurrent state. A batch with multi-token portions reads the carried rows from a copy
taken at its start, because a portion's first and last rows are handled by different workgroups.
"""
from __future__ import annotations

import numpy as np
import torch
import torch.nn.functional as F

from ..models.hybrid_config import DiffAttentionSpec
from ..ops import diff_attention as da
from ..ops import gated_scan as gs
from ..ops import moe
from ..ops import skinny_mm as smm
from ..ops.gemv import skinny_linear
from ..ops.rms_shift import Branch, rms_shift
from .runner import KVCache, SlotState, StepRunner

SPLIT_CLOSE = (1024, 4096)  # rows between which the closing product runs as two (HybridRunner._close)
SKINNY_M = 16   # rows up to which projections stream on the skinny matrix-core kernel


class _Batch:
    """Device-side description of a step. ``single``: every entry is one token (the decode step)."""

    def __init__(self, tokens, pos, slots, max_kv):
        self.tokens, self.pos, self.slots, self.max_kv = tokens, pos, slots, max_kv
        self.T = tokens.shape[0]
        self.single = True
        self.flags = self.entry = self.tiles = self.row_of = self.rows_all = self.chunks = self.entry_slots = None
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
        self.heads, shapes, widths = {}, [], {"shift": (cfg.n_layers, d)}
        for i, L in enumerate(model.layers):  # layer -> its cache index / its state's name
            if L.attention:
                mx = L.spec.mixer
                sp = da.DiffHeads(mx.heads, mx.kv_heads, mx.dim, mx.vdim, mx.scale, L.lam_value(), 1.0 - mx.diff,
                                  cfg.norm_eps, mx.temp_coef, mx.temp_every)
                self.heads[i] = (len(shapes), sp)
                shapes.append((2 * mx.kv_heads, mx.dim, mx.kv_heads, mx.vdim))
            else:
                widths[f"scan{i}"] = (1, L.spec.mixer.width)
        self.cache = KVCache(len(shapes), max_slots, 0, self.max_len, 0, self.device, self.dtype, page_size=page_size,
                             n_pages=kv_pages, layer_shapes=shapes)
        self.state = SlotState(max_slots, widths, self.device)
        if self.device.type == "cuda":
            from ..utils import tunable
            tunable.ensure(tunable.DECODE_FILE)

    # ---------------------------------------------------------------- linear
    def _linear(self, x, w, out=None, act: int = 0):
        """x W^T (act 2: exact GELU). Few bf16 rows stream the weight on the GEMV / skinny matrix-core kernels."""
        T = x.shape[0]
        if (x.is_cuda and x.dtype == torch.bfloat16 and T <= SKINNY_M and w.shape[0] % 4 == 0 and smm.supported(x, w)
                and (out is None or (out.data_ptr() % 16 == 0 and out.stride(0) % 8 == 0))):
            if out is None:
                out = torch.empty(T, w.shape[0], device=x.device, dtype=x.dtype)
            if T == 1:
                return skinny_linear(x, w, None, act, out=out)
            return smm.mm(x, w, None, act, out=out, packed=self._packed_w(w))
        y = F.linear(x, w)
        if act:
            return moe.act_rows(y, torch.empty_like(y) if out is None else out, gated=False)
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
        """Logits of the rows in ``want`` (None: every row)."""
        m, cfg = self.model, self.cfg
        T, d = b.T, cfg.hidden
        x, branch = None, None
        shift = self.state["shift"]
        carry = None if b.single else shift[:, b.entry_slots]
        for i, L in enumerate(m.layers):
            src = {"embed": m.wte, "tokens": b.tokens} if i == 0 else {}
            x, h, hs = rms_shift(x, branch, cfg.residual_mult, L.norm, cfg.norm_eps, shift=L.shift,
                                 prev=shift[i] if b.single else carry[i], prev_idx=b.slots if b.single else b.entry,
                                 pos=b.pos, flags=b.flags, state=shift[i], slots=b.slots, **src)
            if layers_out is not None and i:
                layers_out.append(x.clone())
            mx = L.spec.mixer
            cols = mx.out_cols
            cat = torch.empty(T, cols + L.ff_cols, device=h.device, dtype=h.dtype)
            mix, up = self._mix_and_up(L, h, hs, cat[:, cols:])
            if L.attention:
                self._attention(i, mix, cat[:, :cols], b)
            elif b.single:
                gs.gated_step(mix, L.b_z, L.b_x, self.state[f"scan{i}"][0], cat[:, :cols], b.pos, b.slots)
            else:
                gs.gated_scan(mix, L.b_z, L.b_x, self.state[f"scan{i}"][0], cat[:, :cols], b.chunks, b.multi)
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
        _, h, _ = rms_shift(x, branch, cfg.residual_mult, m.final_norm, cfg.norm_eps, rows=want, keep_x=False)
        return self._linear(h, m.head)

    def _attention(self, i, qkv, out, b: _Batch):
        ci, sp = self.heads[i]
        kc, vc, tbl = self.cache.k[ci], self.cache.v[ci], self.cache.table
        a = (sp, qkv, kc, vc, tbl, b.pos, b.slots)
        if b.single:
            da.attend_rows(*a, out, b.max_kv, fused_append=True, ws=b.bufs.get("ws"), cnt=b.bufs.get("cnt"))
            return
        da.append(*a)
        if out.is_cuda and da.tiles_ok(sp, out.dtype, self.cache.page_size, out.stride(0)):
            if b.tiles is not None:
                da.attend_tiles(*a, out, b.tiles)
            if b.row_of is not None:
                da.attend_rows(*a, out, b.row_kv, fused_append=False, row_of=b.row_of)
        else:
            da.attend_rows(*a, out, b.max_kv, fused_append=False)

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
        wsf = cnt = 1
        for _, sp in self.heads.values():
            _, _, w, c = da.rows_plan(sp, Bb, Kb, self.dtype)
            wsf, cnt = max(wsf, w), max(cnt, c)
        return {"ws": torch.empty(wsf, device=self.device, dtype=torch.float32),
                "cnt": torch.zeros(cnt, device=self.device, dtype=torch.int32)}

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
