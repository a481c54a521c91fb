"""Decode engine for decoders that are described layer by layer: a list of layers, each with a mixer and possibly a
feed-forward of ``tah_amd.mixers``, norms on the sublayers' outputs and possibly in front of them, and a float32 residual
stream.  Layers may share their weights; caches and states are each layer's own.

:class:`StackEngine` is a :class:`tah_amd.engine.DecodeEngine`: the generation state, sampling, loop and captured step
are the ones every model uses.  Sequences live in slots (``tah_amd.kv_cache.SlotPool``); what a slot holds -- latent
rings, recurrent states -- belongs to the layers.  ``extend`` runs any mix of portions of any slots from where they stand:
prompts, parts of prompts, single tokens; ``prefill`` is ``extend`` of one prompt per slot, and a generation step is the
single-token form of all slots.  A position's logits do not depend on how its sequence was cut into portions or on what
else ran with it, beyond rounding.
"""
from __future__ import annotations

import dataclasses
from typing import Dict, List, Optional, Sequence, Tuple

import torch

from . import ops
from ._capi import TahDuoError
from .engine import DecodeEngine
from .kv_cache import InputTail, SlotPool
from .mixers import Linear, LatentAttention, Step, Sublayer, pad_to, padded
from .ops import _call


@dataclasses.dataclass
class StackLayer:
    mixer: object                       # DeltaMixer, LatentAttention, ...
    coef1: torch.Tensor                 # float32 [cols]: the mixer's output norm and layer scale
    mlp: object = None                  # DenseMlp, MoeMlp, or None
    coef2: Optional[torch.Tensor] = None
    pre1: Optional[torch.Tensor] = None  # float32 [cols]: norm in front of the mixer (None: it reads the residual stream) ...
    pre2: Optional[torch.Tensor] = None  # ... and of the feed-forward
    conv1: Optional[torch.Tensor] = None  # float32 [taps, cols], with pre1: short convolution added to the mixer's input


@dataclasses.dataclass(frozen=True)
class Columns:
    """Where a row's entries lie when norms run over ``groups`` equal groups of them: every group padded to whole units of
    eight columns, all of them to whole steps of 32."""
    width: int
    groups: int = 1

    def __post_init__(self):
        if self.groups < 1 or self.width % self.groups:
            raise TahDuoError(f"a width of {self.width} does not divide into {self.groups} groups")

    @property
    def group_cols(self) -> int:
        return pad_to(self.width // self.groups, 8) if self.groups > 1 else self.cols

    @property
    def cols(self) -> int:
        return pad_to(self.groups * pad_to(self.width // self.groups, 8) if self.groups > 1 else self.width)

    def spread(self, t: torch.Tensor, dim: int = -1) -> torch.Tensor:
        """t with ``width`` entries along ``dim`` -> with ``groups * group_cols``, every group followed by its padding."""
        n = self.width // self.groups
        if self.groups == 1 or n == self.group_cols:
            return t
        t = t.movedim(dim, -1)
        out = torch.zeros(*t.shape[:-1], self.groups, self.group_cols, dtype=t.dtype, device=t.device)
        out[..., :n] = t.reshape(*t.shape[:-1], self.groups, n)
        return out.flatten(-2).movedim(-1, dim).contiguous()

    def gather(self, x: torch.Tensor) -> torch.Tensor:
        """The entries of padded rows."""
        if self.groups == 1:
            return x[..., :self.width]
        return x[..., :self.groups * self.group_cols].unflatten(-1, (self.groups, -1))[..., :self.width // self.groups].flatten(-2)


@dataclasses.dataclass
class StackModel:
    """Weights of such a decoder, padded and re-ordered for the kernels."""
    width: int
    vocab: int
    eps: float
    embed: torch.Tensor                 # element type [vocab, cols]
    head: Linear                        # [vocab padded, cols]
    final_coef: torch.Tensor            # float32 [cols]
    layers: List[StackLayer]
    groups: int = 1                     # of columns that are divided by a root mean square of their own
    embed_scale: float = 1.0

    @property
    def columns(self) -> Columns:
        return Columns(self.width, self.groups)

    @property
    def cols(self) -> int:
        return self.embed.shape[1]

    @property
    def dtype(self) -> torch.dtype:
        return self.embed.dtype


def norm_coef(weight: torch.Tensor, scale: Optional[torch.Tensor], cols: int, zero_centred: bool = True) -> torch.Tensor:
    """What a norm multiplies the divided row by, with a layer scale in it: float32, padded with zeros."""
    c = weight.float() + 1.0 if zero_centred else weight.float()
    if scale is not None:
        c = c * scale.float()
    return padded(c[None], 1, cols)[0].contiguous()


def make_head(w: torch.Tensor, cols: int) -> Linear:
    return Linear(padded(w, pad_to(w.shape[0]), cols))


@dataclasses.dataclass
class _Bound:
    mixer: object
    mlp: object
    conv: object = None


class StackEngine(DecodeEngine):
    def __init__(self, model: StackModel, batch: int, max_len: int, *, device="cuda", slots: Optional[int] = None):
        """``batch`` sequences of at most ``max_len`` tokens.  The element type is the model's."""
        self.cfg = self.w = model
        self.dtype = model.dtype
        self.packed = self.dtype == torch.bfloat16
        if not self.packed and torch.get_float32_matmul_precision() != "highest":
            raise TahDuoError("a float32 model needs float32 matrix products (torch.set_float32_matmul_precision('highest'))")
        self._init_generation(batch, max_len, device)
        dev = self.device
        self.pool = SlotPool(batch, max_len)
        self._positions_on_device = False  # a generation advanced the slots; the pool learns of it when asked next
        self._rope: Dict[tuple, tuple] = {}
        self.bound: List[_Bound] = []
        for i, L in enumerate(model.layers):
            self.binding = i
            self.bound.append(_Bound(None, None))
            self.bound[i].mixer = L.mixer.bind(self)
            self.bound[i].mlp = L.mlp.bind(self) if L.mlp is not None else None
            if L.conv1 is not None:
                tail = InputTail(self.B, L.conv1.shape[0], model.cols, device=dev, dtype=self.dtype)
                self.bound[i].conv = ops.lib().InputConv(L.conv1, tail.rows)
        cols = model.cols
        self.normed = any(L.pre1 is not None for L in model.layers)  # sublayers read norms of the residual stream
        if any((L.pre1 is None) == self.normed or (L.mlp is not None and (L.pre2 is None) == self.normed) for L in model.layers):
            raise TahDuoError("either every sublayer has a norm in front of it or none has")
        self.group = min(batch, ops.LINEAR_MAX_ROWS)  # rows of a single-token pass
        z = lambda *s, dt=torch.float32: torch.zeros(*s, dtype=dt, device=dev)
        i32 = lambda: z(batch, dt=torch.int32)
        self.x = z(batch, cols)
        self.xe = z(batch, cols, dt=self.dtype) if self.packed or self.normed else self.x
        self.slot, self.qpos, self.act = i32(), i32(), z(batch, dt=torch.bool)
        self.xp = z(32 * cols, dt=self.dtype) if self.packed else None
        self.hp = z(32 * cols, dt=self.dtype) if self.packed else None
        self.h = z(batch, cols, dt=self.dtype)
        self.logits = z(batch, model.head.n, dt=self.dtype)
        # single tokens outside a generation (the generation's own state stays as it is)
        self.one_tok, self.one_pos, self.one_off = z(batch, dt=torch.long), i32(), z(batch, dt=torch.bool)

    # ── what layers ask for while they are bound ─────────────────────────
    def ring_of(self, i: int) -> int:
        """The layer whose latents layer i reads."""
        s = self.cfg.layers[i].mixer.spec.source
        return i if s is None else s

    def rope(self, base: float, dims: int) -> Tuple[torch.Tensor, torch.Tensor]:
        """cos / sin float32 [max_len, dims / 2] of position * base^(-2 i / dims)."""
        key = (base, dims)
        if key not in self._rope:
            f = base ** (-torch.arange(0, dims, 2, dtype=torch.float64) / max(dims, 1))
            a = torch.arange(self.max_len, dtype=torch.float64)[:, None] * f[None]
            self._rope[key] = tuple(t.float().contiguous().to(self.device) for t in (a.cos(), a.sin()))
        return self._rope[key]

    # ── layers ───────────────────────────────────────────────────────────
    def _front(self, i: int):
        """(norm, convolution, whether it is the output norm) between the residual stream and layer i's mixer, or behind the
        last layer the output head."""
        m = self.cfg
        return (m.final_coef, None, True) if i == len(m.layers) else (m.layers[i].pre1, self.bound[i].conv, False)

    def _add(self, st: Step, r: Sublayer, coef: Optional[torch.Tensor], front: tuple, h: torch.Tensor) -> None:
        """A sublayer's result into the residual stream, and from it what the next sublayer (or the output head) reads."""
        m, (norm, conv, last) = self.cfg, front
        geometry = (m.groups, m.columns.group_cols)
        args = (st.x, coef, m.width, m.eps, r.y, r.y_scale, r.experts, r.index, r.weight)
        tail = (r.index_scale, r.index_row, *geometry)
        if last:
            _call("residual_norm", *args, None, None, norm, None if st.packed else h, self.hp if st.packed else None, *tail, None, None, None)
        elif norm is None:  # (in float32 the element-type rows are the residual rows themselves)
            _call("residual_norm", *args, st.xe if self.packed and not st.packed else None, st.xp, None, None, None, *tail, None, None, None)
        elif conv is None or st.slot is not None:
            _call("residual_norm", *args, None, None, norm, st.xe, st.xp, *tail, conv, st.slot if conv else None, st.pos if conv else None)
        else:
            n = torch.empty_like(st.xe)
            _call("residual_norm", *args, None, None, norm, n, None, *tail, None, None, None)
            _call("conv_rows", n, conv, st.portions, st.xe)

    def _layers(self, st: Step, h: torch.Tensor, trace: Optional[list] = None) -> None:
        """All layers on the step's rows; the output norm's rows go to ``h`` (or, packed, to ``self.hp``)."""
        single = st.slot is not None
        st.normed = self.normed
        if st.normed:
            self._add(st, Sublayer(), None, self._front(0), h)
        for i, (L, b) in enumerate(zip(self.cfg.layers, self.bound)):
            r = b.mixer.rows(st) if single else b.mixer.portions(st)
            self._add(st, r, L.coef1, self._front(i + 1) if b.mlp is None else (L.pre2, None, False), h)
            if b.mlp is not None:
                r = b.mlp.rows(st) if single else b.mlp.portions(st)
                self._add(st, r, L.coef2, self._front(i + 1), h)
            if trace is not None:
                trace.append(self.cfg.columns.gather(st.x).clone())

    def _single(self, tok, pos, finished) -> torch.Tensor:
        """One token per slot (rows of finished slots are dropped): logits [B, vocab].  Nothing is read by the host."""
        m = self.cfg
        for a in range(0, self.B, self.group):
            b = min(a + self.group, self.B)
            sl = slice(a, b)
            _call("embed_rows", tok[sl], m.embed, self.x[sl], None, None if self.normed else self.xp, pos[sl], finished[sl], self.slot[sl], self.qpos[sl],
                  self.act[sl], a, m.embed_scale)
            st = Step(self.x[sl], self.xe[sl], self.qpos[sl], self.xp, slot=self.slot[sl])
            self._layers(st, self.h[sl])
            if self.packed:
                m.head.rows(self.hp, b - a, out=self.logits[sl])
            else:
                m.head(self.h[sl], out=self.logits[sl])
        return self.logits[:, :m.vocab]

    def _portions(self, slots: Sequence[int], lens: Sequence[int], starts: Sequence[int], ids: torch.Tensor, want: Optional[Sequence[int]],
                  trace: Optional[list] = None):
        """Portions (packed rows) -> logits [len(want), vocab] of the wanted rows."""
        m, dev, N = self.cfg, self.device, int(ids.numel())
        cu = [0]
        for n in lens:
            cu.append(cu[-1] + n)
        # one small upload: boundaries, slots, first positions, rows' sequences and positions, wanted rows
        seq = [b for b, n in enumerate(lens) for _ in range(n)]
        pos = [p for n, s in zip(lens, starts) for p in range(s, s + n)]
        want = list(range(N)) if want is None else list(want)
        meta = torch.tensor(cu + list(slots) + list(starts) + seq + pos + want, dtype=torch.int32).to(dev)
        cu_d, slot_d, start_d, seq_d, pos_d, want_d = (t.contiguous() for t in meta.split([len(cu), len(lens), len(lens), N, N, len(want)]))
        x = torch.empty(N, m.cols, dtype=torch.float32, device=dev)
        xe = torch.empty(N, m.cols, dtype=self.dtype, device=dev) if self.packed or self.normed else x
        _call("embed_rows", ids, m.embed, x, xe if self.packed and not self.normed else None, None, None, None, None, None, None, 0, m.embed_scale)
        st = Step(x, xe, pos_d, portions=ops.lib().Portions(cu_d, slot_d, start_d, seq_d), starts=list(zip(lens, starts)))
        h = torch.empty(N, m.cols, dtype=self.dtype, device=dev)
        self._layers(st, h, trace)
        if not want:
            return torch.empty(0, m.vocab, dtype=self.dtype, device=dev)
        return m.head(h.index_select(0, want_d))[:, :m.vocab]

    # ── sequences ────────────────────────────────────────────────────────
    def alloc(self) -> int:
        """A free slot."""
        return self.pool.alloc()

    def release(self, slot: int) -> None:
        """Gives a sequence's slot back.  (What it holds is not read again: the next sequence starts at position 0.)"""
        self.pool.release(slot)

    def _sync_positions(self) -> None:
        if self._positions_on_device:
            for s, n in enumerate(self.pos.tolist()):
                self.pool.length[s] = n
            self._positions_on_device = False

    @torch.no_grad()
    def extend(self, entries: Sequence[Tuple[int, Sequence[int]]], want: Optional[Sequence[Sequence[int]]] = None,
               trace: Optional[list] = None) -> torch.Tensor:
        """Runs the next tokens of some sequences: ``entries`` lists (slot, tokens), every slot at most once.  ``want``: per
        entry the places among its tokens whose logits are asked for (default: all).  Returns the logits [wanted, vocab] in
        that order.  Entries of one token run in the single-token form, the others as packed portions.  ``trace``: a list
        that receives the residual stream after every layer (of the portions)."""
        self._sync_positions()
        if len({s for s, _ in entries}) != len(entries):
            raise TahDuoError("extend: a slot is listed twice")
        for s, t in entries:
            if not 0 <= s < self.B or not len(t):
                raise TahDuoError("extend: a slot outside the engine, or no tokens for it")
            if self.pool.length[s] + len(t) > self.max_len:
                raise TahDuoError(f"extend: slot {s} would outgrow the cache capacity of {self.max_len}")
        if want is None:
            want = [range(len(t)) for _, t in entries]
        starts = [self.pool.grow(s, len(t)) for s, t in entries]
        ones = [i for i, (_, t) in enumerate(entries) if len(t) == 1]
        many = [i for i, (_, t) in enumerate(entries) if len(t) > 1]
        got: Dict[int, torch.Tensor] = {}
        if many:
            lens = [len(entries[i][1]) for i in many]
            ids = torch.tensor([int(t) for i in many for t in entries[i][1]], dtype=torch.long).to(self.device)
            rows, at = [], 0
            for i, n in zip(many, lens):
                rows += [at + int(k) for k in want[i]]
                at += n
            lg = self._portions([entries[i][0] for i in many], lens, [starts[i] for i in many], ids, rows, trace)
            at = 0
            for i in many:
                got[i] = lg[at:at + len(want[i])]
                at += len(want[i])
        if ones:
            tok, pos, off = [0] * self.B, [0] * self.B, [True] * self.B
            for i in ones:
                s = entries[i][0]
                tok[s], pos[s], off[s] = int(entries[i][1][0]), starts[i], False
            self.one_tok.copy_(torch.tensor(tok))
            self.one_pos.copy_(torch.tensor(pos, dtype=torch.int32))
            self.one_off.copy_(torch.tensor(off))
            lg = self._single(self.one_tok, self.one_pos, self.one_off)
            for i in ones:
                got[i] = lg[entries[i][0]:entries[i][0] + 1].clone() if len(want[i]) else lg[:0]
        return torch.cat([got[i] for i in range(len(entries))])

    @torch.no_grad()
    def prefill(self, ids: torch.Tensor, cu: torch.Tensor, *, portion: Optional[int] = None):
        """A new batch, one prompt per slot: ids int64 [N] (the prompts one after another), cu int32 [B + 1].  Returns the
        logits float32 [B, vocab] of each prompt's last token and None (no token takes a second iteration).  ``portion``:
        at most so many tokens of a prompt per pass (bounds the memory of long prompts)."""
        cu_h = cu.cpu().tolist()
        if len(cu_h) != self.B + 1:
            raise TahDuoError("cu must have batch + 1 entries")
        lens = [b - a for a, b in zip(cu_h, cu_h[1:])]
        if min(lens) < 1 or max(lens) > self.max_len:
            raise TahDuoError("a prompt is empty or longer than the cache capacity")
        self.pool.take_all()
        self._positions_on_device = False
        self.n_hard.zero_()
        self.n_steps.zero_()
        self._graph = None
        step = portion or max(lens)
        first = torch.empty(self.B, self.cfg.vocab, dtype=torch.float32, device=self.device)
        for at in range(0, max(lens), step):
            live = [b for b in range(self.B) if lens[b] > at]
            part = [min(step, lens[b] - at) for b in live]
            rows, r = [], 0
            done = []
            for b, n in zip(live, part):
                r += n
                if at + n == lens[b]:
                    rows.append(r - 1)
                    done.append(b)
            seg = ids if len(live) == self.B and step >= max(lens) else torch.cat([ids[cu_h[b] + at:cu_h[b] + at + n] for b, n in zip(live, part)])
            lg = self._portions(live, part, [self.pool.grow(b, n) for b, n in zip(live, part)], seg.contiguous(), rows)
            if done:
                first[torch.tensor(done, device=self.device)] = lg.float()
        self.pos.copy_(torch.tensor(lens, dtype=torch.int32))
        self.host_positions = max(lens)
        self.finished.zero_()
        return first, None

    # ── generation (DecodeEngine) ────────────────────────────────────────
    def _parts(self):
        return self._single(self.tok, self.pos, self.finished), None, None, ~self.finished

    def _advanced(self, steps: int) -> None:
        super()._advanced(steps)
        self._positions_on_device = True

    def _hold_state(self):
        state = [t.clone() for t in self._state()]
        self.finished.fill_(True)  # every row dropped: a warm-up step touches no slot

        def undo():
            for t, old in zip(self._state(), state):
                t.copy_(old)
        return undo
