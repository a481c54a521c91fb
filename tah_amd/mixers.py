"""Layer mechanisms of decoders that are described layer by layer, each a class over the kernels of
include/tah_mixers.h with its sizes and constants as parameters: a mixer (gated delta rule, latent attention, attention in a
window with kept first tokens) and a feed-forward (dense, mixture of experts).  ``tah_amd.stack`` puts them together.

Every mechanism runs in two forms.  ``portions(step)``: rows of several tokens per sequence (prompts, parts of prompts),
with library GEMMs for the dense products.  ``rows(step)``: one token per sequence, at most 32 rows; in bf16 the dense
products run on ``ops.linear_rows`` from re-ordered weights and hand their results on in operand order.  In float32
(a model's exact form) both use library GEMMs.

Sizes are padded where the weights are loaded (``pad_to``), with zeros: the matrix kernels then see whole steps of 32
whatever a model's sizes are.
"""
from __future__ import annotations

import dataclasses
import math
from typing import Dict, Optional, Tuple

import torch

from . import ops
from ._capi import TahDuoError
from .kv_cache import LatentRing, RecurrentState, WindowCache
from .ops import _call


@dataclasses.dataclass(frozen=True)
class Activation:
    """An element-wise function of a feed-forward's hidden rows: ``kind`` and constants for ``activate_rows``, and the keyword
    that makes it the epilogue of ``ops.linear_rows``."""
    kind: int
    c: Tuple[float, float] = (0.0, 0.0)
    rows: Dict[str, object] = dataclasses.field(default_factory=dict)

    def __call__(self, h: torch.Tensor, out: Optional[torch.Tensor] = None) -> torch.Tensor:
        return _call("activate_rows", h, self.kind, out, *self.c)


GELU_TANH = Activation(0, rows={"gelu_tanh": True})
SILU_MUL = Activation(1)


def softplus(x: float) -> float:
    return max(x, 0.0) + math.log1p(math.exp(-abs(x)))


def xielu(p: float, q: float) -> Activation:
    """softplus(p) x^2 + x / 2 above zero, (1/2 + softplus(q)) (exp(x) - 1 - x) + x / 2 below."""
    c = (softplus(p), 0.5 + softplus(q))
    return Activation(2, c, {"xielu": c})


def clamped_gate(limit: float, slope: float = 1.702) -> Activation:
    """g sigmoid(slope g) (u + 1) of g = min(gate, limit) and u = up cut off at both limits."""
    c = (limit, slope)
    return Activation(3, c, {"clamped": c})


def pad_to(n: int, m: int = 32) -> int:
    return (n + m - 1) // m * m


def padded(w: torch.Tensor, rows: int, cols: int) -> torch.Tensor:
    """w [r, c] in the upper left corner of zeros [rows, cols]."""
    out = torch.zeros(rows, cols, dtype=w.dtype, device=w.device)
    out[:w.shape[0], :w.shape[1]] = w
    return out


def padded_heads(w: torch.Tensor, heads: int, size: int, to: int) -> torch.Tensor:
    """w [heads * size, c] -> [heads * to, c], each head's rows followed by zero rows."""
    out = torch.zeros(heads, to, w.shape[1], dtype=w.dtype, device=w.device)
    out[:, :size] = w.view(heads, size, w.shape[1])
    return out.view(heads * to, w.shape[1])


class Linear:
    """A dense layer, weight [n, k] with both sizes whole steps of 32."""

    def __init__(self, w: torch.Tensor):
        self.w = w.contiguous()
        self.n, self.k = self.w.shape
        self.packed = ops.linear_pack_weight(self.w) if w.dtype == torch.bfloat16 else None

    def __call__(self, x: torch.Tensor, out: Optional[torch.Tensor] = None) -> torch.Tensor:
        return torch.matmul(x, self.w.t(), out=out) if out is not None else x @ self.w.t()

    def rows(self, xp: torch.Tensor, rows: int, **kw):
        return ops.linear_rows(self.packed, xp, rows, self.n, self.k, **kw)


class PackedBatch:
    """Weights of several products of the same sizes, [batch, n, k], for one ``ops.linear_rows`` launch."""

    def __init__(self, w: torch.Tensor, gate_up: bool = False):
        self.batch, n, self.k = w.shape
        self.n = n // 2 if gate_up else n
        self.gate_up = gate_up
        self.w = torch.cat([ops.linear_pack_weight(x.contiguous(), gate_up=gate_up) for x in w])

    def rows(self, xp: torch.Tensor, rows: int, **kw):
        return ops.linear_rows(self.w, xp, rows, self.n, self.k, gate_up=self.gate_up, batch=self.batch, **kw)


@dataclasses.dataclass
class Step:
    """What a forward of some rows carries through the layers.  x float32 [rows, cols] is the residual stream, xe what the next
    sublayer reads, in the element type (the same rows, or with ``normed`` the norm in front of it), xp (bf16, at most 32
    rows) its rows form; the rest says whose rows they are."""
    x: torch.Tensor
    xe: torch.Tensor
    pos: torch.Tensor                          # int32 [rows]
    xp: Optional[torch.Tensor] = None
    slot: Optional[torch.Tensor] = None        # one token per row: slots (negative: dropped)
    portions: object = None                    # several tokens per sequence: tah_amd._C.Portions ...
    starts: Optional[list] = None              # ... and on the host: (length, first position) per sequence
    contexts: Dict[int, tuple] = dataclasses.field(default_factory=dict)  # latent rows portions can see, per ring
    normed: bool = False

    @property
    def n(self) -> int:
        return self.x.shape[0]

    @property
    def packed(self) -> bool:
        return self.xp is not None


@dataclasses.dataclass
class Sublayer:
    """A sublayer's result on its way to the residual sum: y (optionally times y_scale per row), and / or expert rows."""
    y: Optional[torch.Tensor] = None
    y_scale: Optional[torch.Tensor] = None
    experts: Optional[torch.Tensor] = None
    index: Optional[torch.Tensor] = None
    weight: Optional[torch.Tensor] = None
    index_scale: int = 1
    index_row: int = 0


# ── gated delta rule ─────────────────────────────────────────────────────────────────────────────────────────────────
@dataclasses.dataclass(frozen=True)
class DeltaSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int
    eps: float

    @property
    def channels(self) -> int:
        return 2 * self.kv_heads * self.dim + self.heads * self.vdim


class DeltaMixer:
    """Gated delta rule with short convolutions.  Weights: q, k, v, g (gate), b (step), a (decay), o projections [out, in],
    conv_q, conv_k, conv_v [channels, taps], a_log, dt_bias [heads], norm [vdim]."""

    def __init__(self, spec: DeltaSpec, w: Dict[str, torch.Tensor], cols: int):
        s = self.spec = spec
        parts = [w[k] for k in ("q", "k", "v", "g", "b", "a")]
        at, self.cols = 0, []
        for p in parts:
            self.cols.append(at)
            at += p.shape[0]
        self.proj = Linear(padded(torch.cat(parts), pad_to(at), cols))
        self.width_o = pad_to(s.heads * s.vdim)
        self.o = Linear(padded(w["o"], cols, self.width_o))
        f = lambda t: t.float().contiguous()
        self.conv = f(torch.cat([w["conv_q"], w["conv_k"], w["conv_v"]]))
        self.a_log, self.dt_bias, self.norm = f(w["a_log"]), f(w["dt_bias"]), f(w["norm"])

    def bind(self, engine) -> "DeltaMixer.Bound":
        return DeltaMixer.Bound(self, engine)

    class Bound:
        """The layer on an engine's slots."""

        def __init__(self, m: "DeltaMixer", engine):
            s = m.spec
            self.m = m
            self.cache = RecurrentState(engine.B, s.heads, s.dim, s.vdim, s.taps, s.channels, device=engine.device, dtype=engine.dtype)
            self.layer = ops.lib().DeltaLayer(m.conv, m.a_log, m.dt_bias, m.norm, self.cache.conv, self.cache.state, s.heads, s.kv_heads,
                                              s.dim, s.vdim, m.cols, s.eps)
            self.op = torch.zeros(32 * m.width_o, dtype=torch.bfloat16, device=engine.device) if engine.packed else None

        def rows(self, st: Step) -> Sublayer:
            m = self.m
            if st.packed:
                proj = m.proj.rows(st.xp, st.n)
                _call_on(self.layer.step, proj, st.slot, st.pos, None, self.op)
                return Sublayer(m.o.rows(self.op, st.n))
            out = torch.empty(st.n, m.width_o, dtype=st.xe.dtype, device=st.x.device)
            _call_on(self.layer.step, m.proj(st.xe), st.slot, st.pos, out, None)
            return Sublayer(m.o(out))

        def portions(self, st: Step) -> Sublayer:
            m = self.m
            out = torch.empty(st.n, m.width_o, dtype=st.xe.dtype, device=st.x.device)
            _call_on(self.layer.portions, m.proj(st.xe), st.portions, out)
            return Sublayer(m.o(out))


# ── latent attention ─────────────────────────────────────────────────────────────────────────────────────────────────
@dataclasses.dataclass(frozen=True)
class LatentSpec:
    heads: int
    dim: int            # unrotated query / key dimensions of a head
    rot_dim: int        # rotated ones
    vdim: int
    rank: int
    rope_base: float
    scale: float
    eps: float
    window: Optional[int] = None     # None: no window
    source: Optional[int] = None     # layer whose latents and rotated key part this layer reads


class LatentAttention:
    """Latent attention.  Weights [out, in]: q (per head dim | rot_dim rows), uk [heads * dim, rank], uv [heads * vdim, rank],
    o, and unless the layer reads another one's latents dkv [rank + rot_dim, width] with dkv_norm [rank].

    Portions expand the latents to keys and values of all heads (two GEMMs over the rows they can see); single tokens
    attend on the cached latents themselves, with the query carried over by uk and the result by uv."""

    def __init__(self, spec: LatentSpec, w: Dict[str, torch.Tensor], cols: int):
        s = self.spec = spec
        H = s.heads
        self.dim_p, self.rot_p, self.rank_p, self.vdim_p = pad_to(s.dim), pad_to(s.rot_dim), pad_to(s.rank), pad_to(s.vdim, 16)
        q = w["q"].view(H, s.dim + s.rot_dim, -1)
        qp = torch.zeros(H, self.dim_p + self.rot_p, q.shape[2], dtype=q.dtype, device=q.device)
        qp[:, :s.dim], qp[:, self.dim_p:self.dim_p + s.rot_dim] = q[:, :s.dim], q[:, s.dim:]
        q = qp.view(H * (self.dim_p + self.rot_p), -1)
        self.owner = s.source is None
        self.dkv_col = q.shape[0] if self.owner else -1
        proj = torch.cat([q, w["dkv"]]) if self.owner else q
        self.proj = Linear(padded(proj, pad_to(proj.shape[0]), cols))
        self.dkv_norm = w["dkv_norm"].float().contiguous() if self.owner else None
        self.width_o = pad_to(H * self.vdim_p)
        uk = padded(padded_heads(w["uk"], H, s.dim, self.dim_p), H * self.dim_p, self.rank_p)
        uv = padded(padded_heads(w["uv"], H, s.vdim, self.vdim_p), H * self.vdim_p, self.rank_p)
        o = padded_heads(w["o"].t().contiguous(), H, s.vdim, self.vdim_p).t()
        self.o = Linear(padded(o, cols, self.width_o))
        self.uk, self.uv = uk.contiguous(), uv.contiguous()
        uk_h, uv_h = uk.view(H, self.dim_p, self.rank_p), uv.view(H, self.vdim_p, self.rank_p)
        self.uk_t = uk_h.transpose(1, 2).contiguous()                     # [H, rank_p, dim_p]
        self.packed = q.dtype == torch.bfloat16
        if self.packed:
            self.uk_rows, self.uv_rows = PackedBatch(self.uk_t), PackedBatch(uv_h)

    def bind(self, engine) -> "LatentAttention.Bound":
        return LatentAttention.Bound(self, engine)

    class Bound:
        def __init__(self, m: "LatentAttention", engine):
            s = m.spec
            self.m, self.engine = m, engine
            if m.owner:
                # as long as the widest window among the layers that read this cache, and no longer than a sequence
                widest = [l.mixer.spec.window for i, l in enumerate(engine.cfg.layers)
                          if isinstance(l.mixer, LatentAttention) and engine.ring_of(i) == engine.binding]
                cap = engine.max_len if None in widest else min(max(widest), engine.max_len)
                self.ring = LatentRing(engine.B, cap, m.rank_p, m.rot_p, device=engine.device, dtype=engine.dtype)
                self.source = engine.binding
            else:
                src = engine.bound[s.source].mixer
                if not isinstance(src, LatentAttention.Bound) or not src.m.owner:
                    raise TahDuoError(f"layer {engine.binding} reads the latents of layer {s.source}, which has none of its own")
                if (src.m.spec.rank, src.m.spec.rot_dim, src.m.spec.rope_base) != (s.rank, s.rot_dim, s.rope_base):
                    raise TahDuoError(f"layers {engine.binding} and {s.source} share latents of different sizes or rotations")
                self.ring, self.source = src.ring, s.source
            cap = self.ring.rows.shape[1]
            self.window = cap if s.window is None else min(s.window, cap)
            self.layer = ops.lib().LatentLayer(self.ring.rows, s.heads, m.dim_p, s.rot_dim, m.rot_p, s.rank, m.rank_p, m.vdim_p, self.window, s.scale)
            self.cos, self.sin = engine.rope(s.rope_base, s.rot_dim)
            z = lambda n, dt=engine.dtype: torch.zeros(n, dtype=dt, device=engine.device)
            self.workspace = z(max(int(self.layer.decode_workspace(min(engine.B, 32))), 16), torch.uint8)
            if engine.packed:
                self.qp, self.cp, self.op = z(s.heads * 32 * m.dim_p), z(s.heads * 32 * m.rank_p), z(32 * m.width_o)

        def _prep(self, proj, st: Step, slot=None, rows_out=None, q_packed=None, q_rows=None):
            m = self.m
            _call_on(self.layer.prep, proj, 0, m.dkv_col, m.dkv_norm, m.spec.eps, self.cos, self.sin, st.pos, slot, rows_out, q_packed, q_rows)

        def rows(self, st: Step) -> Sublayer:
            m, H, n = self.m, self.m.spec.heads, st.n
            if st.packed:
                proj = m.proj.rows(st.xp, n)
                self._prep(proj, st, slot=st.slot, q_packed=self.qp)
                q = m.uk_rows.rows(self.qp, n)   # [H, n, rank_p]
                _call_on(self.layer.decode, st.slot, st.pos, q, proj, 0, self.cp, None, self.workspace)
                m.uv_rows.rows(self.cp, n, out_packed=self.op, want_out=False, packed_col_step=m.vdim_p)
                return Sublayer(m.o.rows(self.op, n))
            e = lambda *shape: torch.empty(*shape, dtype=st.xe.dtype, device=st.x.device)
            proj, q_rows, c_rows = m.proj(st.xe), e(H, n, m.dim_p), e(H, n, m.rank_p)
            self._prep(proj, st, slot=st.slot, q_rows=q_rows)
            q = torch.matmul(q_rows, m.uk.view(H, m.dim_p, m.rank_p))
            _call_on(self.layer.decode, st.slot, st.pos, q, proj, 0, None, c_rows, self.workspace)
            y = torch.matmul(c_rows, m.uv.view(H, m.vdim_p, m.rank_p).transpose(1, 2).contiguous())   # [H, n, vdim_p]
            out = torch.zeros(n, m.width_o, dtype=st.xe.dtype, device=st.x.device)
            out[:, :H * m.vdim_p] = y.transpose(0, 1).reshape(n, -1)
            return Sublayer(m.o(out))

        def portions(self, st: Step) -> Sublayer:
            m, H, n = self.m, self.m.spec.heads, st.n
            e = lambda *shape: torch.empty(*shape, dtype=st.xe.dtype, device=st.x.device)
            proj = m.proj(st.xe)
            if m.owner:
                new = e(n, m.rank_p + m.rot_p)
                self._prep(proj, st, rows_out=new)
                # what the portions can see: their own rows and what the ring still holds of the rows before them
                cap, cu = self.ring.rows.shape[1], [0]
                for length, first in st.starts:
                    cu.append(cu[-1] + length + min(first, cap - 1))
                cu_k = torch.tensor(cu, dtype=torch.int32).to(st.x.device)
                ctx = e(cu[-1], m.rank_p + m.rot_p)
                _call_on(self.layer.context, st.portions, cu_k, new, ctx)
                st.contexts[self.source] = (ctx, cu_k)
            else:
                self._prep(proj, st)
                ctx, cu_k = st.contexts[self.source]
            c = ctx[:, :m.rank_p]
            out = e(n, m.width_o) if m.width_o == H * m.vdim_p else torch.zeros(n, m.width_o, dtype=st.xe.dtype, device=st.x.device)
            _call_on(self.layer.attend, st.portions, cu_k, max(l for l, _ in st.starts), proj, 0, c @ m.uk.t(), c @ m.uv.t(), ctx, out)
            return Sublayer(m.o(out))


# ── attention in a window with kept first tokens ─────────────────────────────────────────────────────────────────────
@dataclasses.dataclass(frozen=True)
class WindowSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    rot_dim: int                     # the first so many dimensions of a head are rotated
    rope_base: float
    scale: float
    window: Optional[int] = None     # position i sees j <= i with i - j < window (None: all) ...
    keep_first: int = 0              # ... or j < keep_first
    adjacent: bool = True            # rotated pairs are dimensions 2 i and 2 i + 1 (else i and i + rot_dim / 2)


class WindowAttention:
    """Attention with grouped query heads in a sliding window that keeps a sequence's first tokens.  Weights [out, in]: q [heads *
    dim, width], k [kv_heads * dim, width], o [width, heads * vdim]; v [kv_heads * vdim, width], or none when the keys before
    their rotation are the values; g [heads, width], or none: a sigmoid gate per head on its result.

    What is cached of a token and key/value head is one row, values in front, keys at its end, rotated dimensions last.
    Without v the two overlap: [rotated dimensions, unrotated | the others | rotated dimensions, rotated], the values
    being the first two parts and the keys the last two.  Queries and the output projection follow that order, which is
    given to the weights here."""

    def __init__(self, spec: WindowSpec, w: Dict[str, torch.Tensor], cols: int):
        s = self.spec = spec
        H, G, D, rd = s.heads, s.kv_heads, s.dim, s.rot_dim
        tied = "v" not in w
        if H % G or rd > D or rd % 2 or (tied and s.vdim != D):
            raise TahDuoError(f"attention: {H} heads on {G}, {rd} of {D} dimensions rotated, values of {s.vdim}: sizes that do not go together")
        self.rot_pad = pad_to(rd, 16)
        self.key_dim = pad_to(self.rot_pad + D - rd)
        rest = self.key_dim - self.rot_pad
        turned = list(range(rd)) if s.adjacent else [i + h * (rd // 2) for i in range(rd // 2) for h in (0, 1)]
        others = list(range(rd, D))
        pad = lambda idx, n: idx + [-1] * (n - len(idx))
        key = pad(others, rest) + pad(turned, self.rot_pad)
        if tied:
            value = pad(turned, self.rot_pad) + pad(others, rest)
            row, self.rot_source = value + [-1] * self.rot_pad, 0
            kv = self._ordered(w["k"], G, D, row)
        else:
            value = pad(list(range(s.vdim)), pad_to(s.vdim))
            row, self.rot_source = value + key, len(value) + rest
            kv = torch.cat([self._ordered(w["v"], G, s.vdim, value).view(G, len(value), -1), self._ordered(w["k"], G, D, key).view(G, len(key), -1)],
                           1).flatten(0, 1)
        self.value_dim, self.row = len(value), len(row)
        parts = [self._ordered(w["q"], H, D, key), kv] + ([w["g"]] if "g" in w else [])
        self.k_col = H * self.key_dim
        self.g_col = self.k_col + G * self.row if "g" in w else -1
        proj = torch.cat(parts)
        self.proj = Linear(padded(proj, pad_to(proj.shape[0]), cols))
        self.width_o = H * self.value_dim
        self.o = Linear(padded(self._ordered(w["o"].t().contiguous(), H, s.vdim, value).t(), cols, self.width_o))

    @staticmethod
    def _ordered(w: torch.Tensor, heads: int, size: int, order: list) -> torch.Tensor:
        """w [heads * size, c] -> [heads * len(order), c]: a head's rows in the given order, zeros for -1."""
        w = w.view(heads, size, -1)
        idx = torch.tensor(order, device=w.device)
        out = w[:, idx.clamp_min(0)]
        out[:, idx < 0] = 0
        return out.flatten(0, 1)

    def bind(self, engine) -> "WindowAttention.Bound":
        return WindowAttention.Bound(self, engine)

    class Bound:
        def __init__(self, m: "WindowAttention", engine):
            s = m.spec
            self.m = m
            keep = min(s.keep_first, engine.max_len)
            window = engine.max_len if s.window is None else min(s.window, engine.max_len)
            self.cache = WindowCache(engine.B, s.kv_heads, keep, window, m.row, device=engine.device, dtype=engine.dtype)
            self.layer = ops.lib().WindowLayer(self.cache.rows, *engine.rope(s.rope_base, s.rot_dim), s.heads, m.key_dim, m.value_dim, s.rot_dim,
                                               m.rot_pad, m.rot_source, keep, window, s.scale, 0, m.k_col, m.g_col)
            z = lambda n, dt=engine.dtype: torch.zeros(n, dtype=dt, device=engine.device)
            self.workspace = z(max(int(self.layer.decode_workspace(min(engine.B, ops.LINEAR_MAX_ROWS))), 16), torch.uint8)
            self.op = z(32 * m.width_o) if engine.packed else None

        def rows(self, st: Step) -> Sublayer:
            m = self.m
            if st.packed:
                _call_on(self.layer.decode, m.proj.rows(st.xp, st.n), st.slot, st.pos, None, self.op, self.workspace)
                return Sublayer(m.o.rows(self.op, st.n))
            out = torch.empty(st.n, m.width_o, dtype=st.xe.dtype, device=st.x.device)
            _call_on(self.layer.decode, m.proj(st.xe), st.slot, st.pos, out, None, self.workspace)
            return Sublayer(m.o(out))

        def portions(self, st: Step) -> Sublayer:
            m = self.m
            out = torch.empty(st.n, m.width_o, dtype=st.xe.dtype, device=st.x.device)
            _call_on(self.layer.portions, m.proj(st.xe), st.portions, st.pos, out)
            return Sublayer(m.o(out))


# ── feed-forward ─────────────────────────────────────────────────────────────────────────────────────────────────────
class DenseMlp:
    """down(act(up(x))).  Weights up [ff, width], down [width, ff].  (act(0) = 0: padding stays zero.)"""

    def __init__(self, w: Dict[str, torch.Tensor], cols: int, act: Activation = GELU_TANH):
        self.act = act
        ff = pad_to(w["up"].shape[0])
        self.up, self.down = Linear(padded(w["up"], ff, cols)), Linear(padded(w["down"], cols, ff))

    def bind(self, engine) -> "DenseMlp.Bound":
        return DenseMlp.Bound(self, engine)

    class Bound:
        def __init__(self, m: "DenseMlp", engine):
            self.m = m
            self.ap = torch.zeros(32 * m.up.n, dtype=torch.bfloat16, device=engine.device) if engine.packed else None

        def rows(self, st: Step) -> Sublayer:
            if not st.packed:
                return self.portions(st)
            self.m.up.rows(st.xp, st.n, out_packed=self.ap, want_out=False, **self.m.act.rows)
            return Sublayer(self.m.down.rows(self.ap, st.n))

        def portions(self, st: Step) -> Sublayer:
            h = self.m.up(st.xe)
            return Sublayer(self.m.down(self.m.act(h, h)))


class GatedMlp:
    """down(silu(gate(x)) * up(x)).  Weights gate, up [ff, width], down [width, ff]."""

    def __init__(self, w: Dict[str, torch.Tensor], cols: int):
        ff = pad_to(w["gate"].shape[0])
        self.gate_up = torch.cat([padded(w["gate"], ff, cols), padded(w["up"], ff, cols)])
        self.ff, self.cols = ff, cols
        self.down = Linear(padded(w["down"], cols, ff))
        self.gate_up_packed = ops.linear_pack_weight(self.gate_up, gate_up=True) if self.gate_up.dtype == torch.bfloat16 else None

    def rows(self, xp: torch.Tensor, n: int, act: torch.Tensor) -> torch.Tensor:
        ops.linear_rows(self.gate_up_packed, xp, n, self.ff, self.cols, gate_up=True, out_packed=act, want_out=False)
        return self.down.rows(act, n)

    def __call__(self, x: torch.Tensor) -> torch.Tensor:
        return self.down(SILU_MUL(x @ self.gate_up.t()))


@dataclasses.dataclass(frozen=True)
class Router:
    """How a token chooses among experts: the ``top`` largest scores, which are the logits (weights: softmax over the chosen
    ones) or with ``sigmoid`` their sigmoids (weights: the chosen scores).  ``groups`` equal groups of neighbours: only the
    ``keep`` groups with the largest sum of their two largest scores can be chosen from."""
    top: int
    sigmoid: bool = False
    groups: int = 1
    keep: int = 1


class MoeMlp:
    """Mixture of gated experts, the router in float32; optionally a shared expert for every token, times sigmoid(gate . x).
    Weights: router [experts, width], gate, up [experts, ff, width], down [experts, width, ff]; shared: dict of a
    GatedMlp's weights and sg [1, width], or None.  ``act``: the experts' gate."""

    def __init__(self, router: Router, w: Dict[str, torch.Tensor], shared: Optional[Dict[str, torch.Tensor]], cols: int, act: Activation = SILU_MUL):
        self.rule, self.act, self.top, self.experts, self.cols = router, act, router.top, w["router"].shape[0], cols
        if self.experts % router.groups or not 0 < router.keep <= router.groups or router.top > self.experts // router.groups * router.keep:
            raise TahDuoError(f"experts: {router.top} of {self.experts} from {router.keep} of {router.groups} groups: sizes that do not go together")
        self.router = padded(w["router"], self.experts, cols)
        E, ff = self.experts, pad_to(w["gate"].shape[1])
        self.ff = ff
        gu = torch.zeros(E, 2 * ff, cols, dtype=self.router.dtype, device=self.router.device)
        f0, c0 = w["gate"].shape[1], w["gate"].shape[2]
        gu[:, :f0, :c0], gu[:, ff:ff + f0, :c0] = w["gate"], w["up"]
        down = torch.zeros(E, cols, ff, dtype=gu.dtype, device=gu.device)
        down[:, :c0, :f0] = w["down"]
        self.gate_up, self.down = gu, down
        if gu.dtype == torch.bfloat16:
            self.gate_up_rows, self.down_rows = PackedBatch(gu, gate_up=True), PackedBatch(down)
        self.shared = GatedMlp(shared, cols) if shared else None
        self.shared_gate = padded(shared["sg"], 1, cols) if shared else None

    def bind(self, engine) -> "MoeMlp.Bound":
        return MoeMlp.Bound(self, engine)

    class Bound:
        def __init__(self, m: "MoeMlp", engine):
            self.m = m
            if engine.packed:
                z = lambda n: torch.zeros(n, dtype=torch.bfloat16, device=engine.device)
                self.ap = z(m.experts * 32 * m.ff)
                self.shared_ap = z(32 * m.shared.ff) if m.shared else None

        def _route(self, st: Step):
            m, dev = self.m, st.x.device
            index = torch.empty(st.n, m.top, dtype=torch.int32, device=dev)
            weight = torch.empty(st.n, m.top, dtype=torch.float32, device=dev)
            sg = torch.empty(st.n, dtype=torch.float32, device=dev) if m.shared else None
            _call("moe_route", st.xe if st.normed else st.x, m.router, m.shared_gate, index, weight, sg, int(m.rule.sigmoid), m.rule.groups, m.rule.keep)
            return index, weight, sg

        def rows(self, st: Step) -> Sublayer:
            m, n = self.m, st.n
            if not st.packed:
                return self.portions(st)
            index, weight, sg = self._route(st)
            # every expert that some row chose, over all rows: at this size a product costs its weights, not its rows
            m.gate_up_rows.rows(st.xp, n, shared_rows=True, out_packed=self.ap, want_out=False, select=index, **m.act.rows)
            y = m.down_rows.rows(self.ap, n, select=index)
            shared = m.shared.rows(st.xp, n, self.shared_ap) if m.shared else None
            return Sublayer(shared, sg, y.view(m.experts * n, m.cols), index, weight, index_scale=n, index_row=1)

        def portions(self, st: Step) -> Sublayer:
            m = self.m
            index, weight, sg = self._route(st)
            source, tiles, place = _call("moe_plan", index, m.experts)
            h = _call("moe_linear", st.xe, m.gate_up, source, tiles, True, "clamped" in m.act.rows, *m.act.c)
            y = _call("moe_linear", h, m.down, source, tiles, False, False, 0.0, 0.0)
            return Sublayer(m.shared(st.xe) if m.shared else None, sg, y, place, weight)


def _call_on(method, *args):
    """A kernel object's method, its errors as the package's own."""
    try:
        return method(*args)
    except RuntimeError as e:
        if isinstance(e, TahDuoError):
            raise
        raise TahDuoError(str(e).split("\nException raised from")[0]) from None
