"""Cases for the layer mechanisms of the Zedudra decoder, on whichever device they are given ("cpu" under the CPU execution
build, "cuda" on the GPU), against oracle/zedudra_ref.py in float64, and small models of it."""
from __future__ import annotations

import copy

import torch

from oracle import zedudra_ref as R
from tests.zozosun_cases import BF, close, i32, portions_of, rnd, unpack_rows


# ── attention in a window with kept first tokens ─────────────────────────────────────────────────────────────────────
def window_of(heads, kv, dim, rot, window, keep, base=50.0, scale=0.4):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": scale, "rot": {"base": base, "dims": rot},
            "mask": {"size": window, "keep_first": keep}}


class Host:
    """What a mechanism asks of the engine it is bound to."""
    from tah_amd.stack import StackEngine
    rope = StackEngine.rope

    def __init__(self, dev, dtype, slots, max_len):
        self.B, self.max_len, self.dtype, self.packed, self.device, self._rope = slots, max_len, dtype, dtype == BF, torch.device(dev), {}


def half_split(x, dims):
    """Rotated pairs (i, i + dims / 2) brought next to each other: the order the oracle rotates."""
    order = [i + h * (dims // 2) for i in range(dims // 2) for h in (0, 1)] + list(range(dims, x.shape[-1]))
    return x[..., order]


def looking_queries(k, heads, m, dtype):
    """Queries that look for one key each: of position p, in turn, for the key at distance size - 1 (the last one inside the
    window), at distance size (the first one outside), the last kept token and the first one behind the kept ones."""
    T, G, D = k.shape
    W, K, base, rd = m["mask"]["size"], m["mask"]["keep_first"], m["rot"]["base"], m["rot"]["dims"]
    q = torch.zeros(T, heads, D, dtype=torch.float64)
    for p in range(T):
        j = (p - (W - 1), p - W, K - 1, K)[p % 4]
        if not 0 <= j <= p:
            continue
        kj = R.rotate_pairs(k[j][None].double(), torch.tensor([j - p]), base, rd)[0]   # the key as seen from p
        kj = kj / kj.pow(2).sum(-1, keepdim=True) * (9.0 / m["scale"])
        q[p] = kj.repeat_interleave(heads // G, 0)
    return q.to(dtype)


def attention_on_rounded(q, k, v, m, dtype):
    """The oracle's attention with queries and keys rounded to the element type after their rotation, as they are cached."""
    pos = torch.arange(q.shape[0])
    qr, kr = (R.rotate_pairs(x, pos, m["rot"]["base"], m["rot"]["dims"]).to(dtype).double() for x in (q, k))
    return R.attention(qr, kr, v, dict(m, rot=dict(m["rot"], dims=0)))


def window_case(dev, dtype, m, total, cuts, steps, stand_out=True, gate=True, own_values=0, adjacent=True, max_len=None, slots=3, seed=6):
    """One sequence next to a shorter one, portions of the given sizes, then single tokens next to a dropped row; twice, the
    second time on the slots and rings of the first.  The layer's input rows hold queries, keys (values) and gates side by
    side, so that the projections only pick them.  ``own_values``: size of values with a projection of their own (0: the
    keys); ``adjacent`` False: rotated pairs half the rotated dimensions apart."""
    from tah_amd import ops
    from tah_amd.mixers import Step, WindowAttention, WindowSpec, pad_to
    H, G, D, W, K = m["heads"], m["kv_heads"], m["dim"], m["mask"]["size"], m["mask"]["keep_first"]
    rd, V = m["rot"]["dims"], own_values or m["dim"]
    parts = {"q": H * D, "k": G * D}
    if own_values:
        parts["v"] = G * V
    if gate:
        parts["g"] = H
    width = max(sum(parts.values()), H * V)
    cols = pad_to(width)
    w, at = {}, 0
    for name, n in parts.items():
        w[name] = torch.eye(width)[at:at + n].to(dtype).to(dev)
        parts[name] = (at, at + n)
        at += n
    w["o"] = torch.eye(width)[:, :H * V].contiguous().to(dtype).to(dev)
    spec = WindowSpec(H, G, D, V, rd, m["rot"]["base"], m["scale"], W, K, adjacent)
    host = Host(dev, dtype, slots, max_len or total + steps)
    layer = WindowAttention(spec, w, cols).bind(host)
    layer.cache.rows.fill_(50.0)
    g = torch.Generator().manual_seed(seed)
    other = max(2, total // 2)
    lens, owner = [total, other], [slots - 1, 0]
    second = [other - 2, 2] if other > 3 else [other]
    seen = {}
    for rerun in range(2):
        xs, want = [], []
        for b, n in enumerate(lens):
            x = rnd(g, n + steps, width).to(dtype)
            pick = lambda name, heads: x[:, slice(*parts[name])].view(n + steps, heads, -1)
            if stand_out and b == 0 and adjacent:
                pick("q", H).copy_(looking_queries(pick("k", G), H, m, dtype))
            q, k = pick("q", H).double(), pick("k", G).double()
            v = pick("v", G).double() if own_values else k
            if not adjacent:
                q, k = half_split(q, rd), half_split(k, rd)
            o = attention_on_rounded(q, k, v, m, dtype)
            sg = R.sigmoid(pick("g", H).double()) if gate else torch.ones(n + steps, H, 1, dtype=torch.float64)
            xs.append(x)
            want.append((o * sg.view(n + steps, H, 1)).reshape(n + steps, H * V))
            seen[b] = (q, k, v, sg.view(n + steps, H, 1))
        rows = lambda b, a, n: torch.nn.functional.pad(xs[b][a:a + n], (0, cols - width))
        got, at = [[], []], [0, 0]
        for i in range(max(len(cuts), len(second))):
            live = [b for b, c in ((0, cuts), (1, second)) if i < len(c)]
            ln = [(cuts, second)[b][i] for b in live]
            xe = torch.cat([rows(b, at[b], n) for b, n in zip(live, ln)]).to(dev)
            P, cu = portions_of(ln, [at[b] for b in live], [owner[b] for b in live], dev)
            pos = i32([p for b, n in zip(live, ln) for p in range(at[b], at[b] + n)], dev)
            y = layer.portions(Step(xe.float(), xe, pos, portions=P, starts=list(zip(ln, [at[b] for b in live])))).y
            for j, b in enumerate(live):
                got[b].append(y[cu[j]:cu[j + 1]])
                at[b] += ln[j]
        for s in range(steps):
            xe = torch.cat([rows(0, total + s, 1), rows(1, other + s, 1), rows(0, 0, 1)]).to(dev)
            st = Step(xe.float(), xe, i32([total + s, other + s, 3], dev), ops.linear_pack_rows(xe) if dtype == BF else None, slot=i32(owner + [-1], dev))
            y = layer.rows(st).y
            assert not y[2].any()
            for b in range(2):
                got[b].append(y[b:b + 1])
        for b in range(2):
            close(torch.cat(got[b])[:, :H * V], want[b], dtype, f"window attention, sequence {b}, run {rerun}")
    assert bool((layer.cache.rows[1] == 50.0).all())  # a slot nobody owned
    if stand_out and adjacent and total + steps >= W + K + 6:  # the edges are in the numbers: one position more or less shows
        q, k, v, sg = seen[0]
        for key in ("size", "keep_first"):
            for d in (-1, 1):
                mm = dict(m, mask=dict(m["mask"], **{key: m["mask"][key] + d}))
                if mm["mask"]["size"] < 1 or mm["mask"]["keep_first"] < 0:
                    continue
                bad = R.attention(q, k, v, mm) - R.attention(q, k, v, m)
                assert float((bad * sg).abs().max()) > 0.3, f"{key} off by {d} does not show"


# ── norms over groups, input convolution ─────────────────────────────────────────────────────────────────────────────
def group_norm_case(dev, dtype, rows, width, groups, top=2, experts=3, seed=7):
    """Norm of a sublayer's output, residual sum, norm of the sum, all over groups of columns of their own size."""
    from tah_amd.ops import _call
    from tah_amd.stack import Columns
    g, at, eps = torch.Generator().manual_seed(seed), Columns(width, groups), 0.03
    cols, scale = at.cols, torch.exp(torch.arange(groups) % 5 * 0.7).repeat_interleave(width // groups)  # groups of unlike sizes
    up = lambda t: torch.nn.functional.pad(at.spread(t), (0, cols - at.spread(t).shape[-1]))
    assert torch.equal(at.gather(up(torch.arange(width)[None])), torch.arange(width)[None])
    x, y, ex = rnd(g, rows, width) * scale, (rnd(g, rows, width) * scale).to(dtype), rnd(g, experts * rows, width).to(dtype)
    idx = torch.stack([torch.randperm(experts, generator=g)[:top] for _ in range(rows)])
    wt, c1, c2 = torch.rand(rows, top, generator=g), 1 + 0.3 * rnd(g, width), 1 + 0.3 * rnd(g, width)
    packed = dtype == BF and rows <= 32
    for use in ("none", "y", "both"):
        s = torch.zeros(rows, width, dtype=torch.float64)
        if use != "none":
            s += y.double()
        if use == "both":
            for r in range(rows):
                for e, p in zip(idx[r].tolist(), wt[r].double()):
                    s[r] += p * ex[e * rows + r].double()
        want = x.double() + (R.group_norm(s, c1.double(), groups, eps) if use != "none" else 0.0)
        xd, n = up(x).to(dev), torch.full((rows, cols), 9.0, dtype=dtype, device=dev)
        xp = torch.zeros(32 * cols, dtype=BF, device=dev) if packed else None
        both = use == "both"
        _call("residual_norm", xd, up(c1[None])[0].to(dev), width, eps, up(y).to(dev) if use != "none" else None, None, up(ex).to(dev) if both else None,
              idx.to(torch.int32).to(dev) if both else None, wt.to(dev) if both else None, None, None, up(c2[None])[0].to(dev), n, xp, rows, 1, groups,
              at.group_cols, None, None, None)
        close(at.gather(xd), want, torch.float32, f"residual, {use}")
        wn = R.group_norm(want, c2.double(), groups, eps)
        close(at.gather(n), wn, dtype, f"norm, {use}", tol=None if dtype == BF else 1e-5)
        assert float(n.float().abs().sum()) == float(at.gather(n).float().abs().sum()) or torch.equal(up(at.gather(n.cpu())), n.cpu())  # padding: zeros
        if packed:
            assert torch.equal(unpack_rows(xp.cpu(), cols)[:rows], n.cpu())
        # one root mean square for all columns is something else
        if groups > 1:
            assert float((R.group_norm(want, c2.double(), 1, eps) - wn).abs().max()) > 0.1


def conv_case(dev, dtype, width, groups, taps, cuts=((5, 2, 9), (1 + 2, 4)), steps=7, seed=8):
    """Input convolution: portions (tah_conv_rows), then single tokens (fused behind the norm), two sequences in the same
    calls, twice on the same slots; a dropped row changes nothing."""
    from tah_amd import ops
    from tah_amd.kv_cache import InputTail
    from tah_amd.ops import _call
    from tah_amd.stack import Columns
    g, at, eps = torch.Generator().manual_seed(seed), Columns(width, groups), 1e-3
    cols = at.cols
    up = lambda t: torch.nn.functional.pad(at.spread(t), (0, cols - at.spread(t).shape[-1]))
    w, coef = rnd(g, width, taps), 1 + 0.3 * rnd(g, width)
    tail = InputTail(4, taps, cols, device=dev, dtype=dtype)
    tail.rows.fill_(77.0)
    conv = ops.lib().InputConv(up(w.t().contiguous()).contiguous().to(dev), tail.rows)
    cd, owner, lens = up(coef[None])[0].contiguous().to(dev), (3, 1), [sum(c) for c in cuts]
    for rerun in range(2):
        x = [rnd(g, n + steps, width) for n in lens]
        h = [R.group_norm(t.double(), coef.double(), groups, eps).to(dtype) for t in x]
        want = [R.add_conv(t.double(), w.double()) for t in h]
        got, done = [[], []], [0, 0]
        for i in range(max(map(len, cuts))):
            live = [b for b in range(2) if i < len(cuts[b])]
            ln = [cuts[b][i] for b in live]
            P, cu = portions_of(ln, [done[b] for b in live], [owner[b] for b in live], dev)
            hd = torch.cat([up(h[b][done[b]:done[b] + n]) for b, n in zip(live, ln)]).to(dev)
            out = torch.full_like(hd, 9.0)
            _call("conv_rows", hd, conv, P, out)
            for j, b in enumerate(live):
                got[b].append(at.gather(out[cu[j]:cu[j + 1]]))
                done[b] += ln[j]
        for s in range(steps):
            rows = torch.stack([x[0][lens[0] + s], x[1][lens[1] + s], x[0][0]])
            xd, out = up(rows).to(dev), torch.full((3, cols), 9.0, dtype=dtype, device=dev)
            xp = torch.zeros(32 * cols, dtype=BF, device=dev) if dtype == BF else None
            _call("residual_norm", xd, None, width, eps, None, None, None, None, None, None, None, cd, out, xp, 1, 0, groups, at.group_cols, conv,
                  i32([*owner, -1], dev), i32([lens[0] + s, lens[1] + s, 2], dev))
            assert torch.equal(xd.cpu(), up(rows))
            if xp is not None:
                assert torch.equal(unpack_rows(xp.cpu(), cols)[:3], out.cpu())
            for b in range(2):
                got[b].append(at.gather(out[b:b + 1]))
        for b in range(2):
            close(torch.cat(got[b]), want[b], dtype, f"convolution of {taps}, sequence {b}")
    assert bool((tail.rows[0] == 77.0).all() and (tail.rows[2] == 77.0).all())


# ── activations, experts ─────────────────────────────────────────────────────────────────────────────────────────────
def activation_case(dev, dtype, rows=5, n=48, k=64, seed=9):
    """xIELU and the clamped gate, on rows of their own and as the last step of a product."""
    from tah_amd import mixers, ops
    g = torch.Generator().manual_seed(seed)
    for p, q in ((0.7, -1.3), (-2.5, 0.4), (30.0, -40.0)):
        act = mixers.xielu(p, q)
        f = lambda z: R.xielu(z, torch.tensor(p, dtype=torch.float64), torch.tensor(q, dtype=torch.float64))
        z = (3 * rnd(g, rows, n)).to(dtype)
        z[0, :4] = torch.tensor([0.0, -20.0, 1e-3, -1e-3])
        close(act(z.to(dev)), f(z.double()), dtype, "xielu")
        small = 0.01 * rnd(g, rows, n)   # what cancels near zero keeps its digits
        if dtype == torch.float32:
            close(act(small.to(dev)), f(small.double()), dtype, "xielu near zero")
        if dtype == BF:
            w, x = (rnd(g, n, k) * k ** -0.5).to(BF), rnd(g, rows, k).to(BF)
            z = x.double() @ w.double().t()
            close(ops.linear_rows(ops.linear_pack_weight(w.to(dev)), ops.linear_pack_rows(x.to(dev)), rows, n, k, **act.rows), f(z), BF, "product, xielu")
    for limit in (0.4, 1.0, 7.0):
        act = mixers.clamped_gate(limit)
        z = (3 * rnd(g, rows, 2 * n)).to(dtype)
        close(act(z.to(dev)), R.clamped_gate(z.double()[:, :n], z.double()[:, n:], limit), dtype, "clamped gate")
        if dtype == BF:
            w, x = (2 * rnd(g, 2 * n, k) * k ** -0.5).to(BF), rnd(g, rows, k).to(BF)
            z = (x.double() @ w.double().t()).to(BF).double()   # (rounded where the product ends)
            y = ops.linear_rows(ops.linear_pack_weight(w.to(dev), gate_up=True), ops.linear_pack_rows(x.to(dev)), rows, n, k, gate_up=True, **act.rows)
            close(y, R.clamped_gate(z[:, :n], z[:, n:], limit), BF, "product, clamped gate")


def moe_case(dev, dtype, rows, width, ff, experts, top, groups, keep, limit, seed=10):
    from tah_amd import ops
    from tah_amd.mixers import MoeMlp, Router, Step, clamped_gate, pad_to
    g = torch.Generator().manual_seed(seed)
    w = {"router": rnd(g, experts, width) * width ** -0.5, "gate": rnd(g, experts, ff, width) * width ** -0.5,
         "up": rnd(g, experts, ff, width) * width ** -0.5, "down": rnd(g, experts, width, ff) * ff ** -0.5}
    w = {k: t.to(dtype) for k, t in w.items()}
    cols = pad_to(width)
    x = rnd(g, rows, width).to(dtype)
    flat = {f"e{e}.{k}": w[k][e].double() for e in range(experts) for k in ("gate", "up", "down")}
    flat["router"] = w["router"].double()
    spec = {"router": {"experts": experts, "top": top, "groups": {"count": groups, "keep": keep}}, "expert": {"limit": limit}}
    want = R.moe_mlp(x.double(), flat, spec)
    idx, p = R.route(x.double(), flat["router"], top, spec["router"]["groups"])
    if keep < groups < experts and rows >= 20:  # the groups matter: without them some token chooses otherwise
        free, _ = R.route(x.double(), flat["router"], top, {"count": 1, "keep": 1})
        assert bool((free.sort(1).values != idx.sort(1).values).any())
    b = MoeMlp(Router(top, True, groups, keep), {k: t.to(dev) for k, t in w.items()}, None, cols, clamped_gate(limit)).bind(Host(dev, dtype, 1, 1))
    xe = torch.nn.functional.pad(x, (0, cols - width)).to(dev)

    def total(r):
        at = r.index.long().cpu() * r.index_scale + torch.arange(rows)[:, None] * r.index_row
        y = (r.experts.double().cpu()[at] * r.weight.double().cpu()[:, :, None]).sum(1)
        assert not y[:, width:].any()
        return y[:, :width]
    st = Step(xe.float(), xe, i32([0] * rows, dev), portions=object(), normed=True)
    index, weight, _ = b._route(st)
    assert torch.equal(index.cpu().long(), idx)
    close(weight, p, torch.float32, "weights")
    close(total(b.portions(st)), want, dtype, "experts, sorted rows")
    if dtype == BF and rows <= 32:
        st = Step(xe.float(), xe, st.pos, ops.linear_pack_rows(xe), slot=st.pos, normed=True)
        close(total(b.rows(st)), want, dtype, "experts, decode rows")


# ── the whole decoder ────────────────────────────────────────────────────────────────────────────────────────────────
def dense_of(ff):
    return {"kind": "dense", "ff": ff}


def moe_of(experts, top, groups, keep, ff, limit):
    return {"kind": "moe", "router": {"experts": experts, "top": top, "groups": {"count": groups, "keep": keep}}, "expert": {"ff": ff, "limit": limit}}


def config(width, vocab, groups, taps, scale, layers, eps=1e-5):
    """``layers``: (mixer, feed-forward), or the number of the layer whose weights this one runs on."""
    out = []
    for l in layers:
        out.append(dict(copy.deepcopy(out[l]), weights_of=l) if isinstance(l, int) else {"type": "attention", "mixer": l[0], "mlp": l[1]})
    return {"architecture": "Zedudra", "width": width, "vocab": vocab, "embedding": {"scale": scale}, "norm": {"eps": eps, "groups": groups},
            "canon": {"taps": taps}, "layers": out}


# sizes that are no multiples of anything, layers on other layers' weights (one of them in front of a layer with weights of its
# own), no feed-forward, nothing kept, a window of one token, every dimension rotated, one expert per token, three taps
ODD = config(44, 61, 4, 3, 2.5, [
    (window_of(3, 1, 20, 6, 5, 3, 100.0, 0.5), moe_of(6, 1, 3, 2, 12, 0.7)),
    (window_of(2, 2, 18, 18, 11, 0, 100.0, 0.6), None),
    0,
    (window_of(4, 2, 12, 2, 1, 2, 30.0, 0.7), dense_of(52)),
    1,
], eps=0.1)
# multiples of the matrix steps, more query heads than one tile takes, heads wider than 128
EVEN = config(96, 128, 3, 4, 9.0, [
    (window_of(8, 4, 32, 16, 9, 4, 10000.0, 0.3), dense_of(160)),
    (window_of(20, 1, 64, 32, 45, 2, 1000.0, 0.25), moe_of(8, 3, 4, 3, 32, 1.5)),
    1,
    (window_of(6, 2, 128, 64, 70, 1, 10000.0, 0.2), None),
    (window_of(2, 1, 160, 32, 21, 6, 500.0, 0.2), moe_of(4, 2, 2, 1, 64, 0.5)),
])
# one group, one tap, every expert open, more kept tokens than the window is long
PLAIN = config(72, 50, 1, 1, 1.0, [
    (window_of(4, 4, 24, 8, 6, 10, 100.0, 0.5), moe_of(5, 2, 1, 1, 20, 2.0)),
    0,
    (window_of(4, 1, 40, 12, 30, 1, 100.0, 0.4), dense_of(64)),
], eps=1e-4)
