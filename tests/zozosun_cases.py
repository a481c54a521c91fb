"""Cases for the layer mechanisms of the Zozosun decoder, on whichever device they are given ("cpu" under the CPU execution
build, "cuda" on the GPU), against oracle/zozosun_ref.py in float64, and small models of it."""
from __future__ import annotations

import torch

from oracle import zozosun_ref as R

BF = torch.bfloat16
DTYPES = {"f32": torch.float32, "bf16": BF}
# largest error of a mechanism's result relative to the result's root mean square: float32 against float64, and with
# operands and results in bf16
TOL = {torch.float32: 2e-5, BF: 3e-2}


def rnd(g, *s):
    return torch.randn(*s, generator=g)


def close(got, want, dtype, what, tol=None):
    got, want = got.detach().double().cpu(), want.double()
    assert got.shape == want.shape, (what, got.shape, want.shape)
    own = 2.0 ** -8 if dtype == BF else 0.0   # rounding of a value itself
    err = float(((got - want).abs() - own * want.abs()).max() / want.pow(2).mean().sqrt().clamp_min(1e-12))
    assert err <= (tol or TOL[dtype]), f"{what}: error {err:.3e} of the result's root mean square (allowed {tol or TOL[dtype]})"
    return err


def unpack_rows(xp, k):
    """Rows form [32 * k] -> [32, k]."""
    return xp.view(k // 32, 2, 4, 16, 8).permute(1, 3, 0, 2, 4).reshape(32, k)


def i32(x, dev):
    return torch.tensor(x, dtype=torch.int32).to(dev)


def portions_of(lens, starts, slots, dev):
    from tah_amd import ops
    cu = [0]
    for n in lens:
        cu.append(cu[-1] + n)
    seq = [b for b, n in enumerate(lens) for _ in range(n)]
    return ops.lib().Portions(i32(cu, dev), i32(slots, dev), i32(starts, dev), i32(seq, dev)), cu


# ── residual rows ────────────────────────────────────────────────────────────────────────────────────────────────────
def rows_case(dev, dtype, rows=5, width=72, cols=96, top=3, experts=4, seed=1):
    from tah_amd.ops import _call
    g = torch.Generator().manual_seed(seed)
    packed = dtype == BF and rows <= 32 and cols % 32 == 0
    z = lambda *s, dt=dtype: torch.zeros(*s, dtype=dt, device=dev)
    pad = lambda t: torch.nn.functional.pad(t, (0, cols - width))
    # tokens into the residual stream; finished rows get no slot
    embed = pad(rnd(g, 11, width)).to(dtype).to(dev)
    tok = torch.randint(0, 11, (rows,), generator=g).to(dev)
    pos, fin = i32(list(range(3, 3 + rows)), dev), torch.tensor([i % 3 == 1 for i in range(rows)]).to(dev)
    x, xe, xp = z(rows, cols, dt=torch.float32), z(rows, cols), (z(32 * cols) if packed else None)
    slot, qpos, act = i32([9] * rows, dev), i32([9] * rows, dev), z(rows, dt=torch.bool)
    _call("embed_rows", tok, embed, x, xe, xp, pos, fin, slot, qpos, act, 7, 1.0)
    assert torch.equal(x, embed[tok].float()) and torch.equal(xe, embed[tok])
    if packed:
        assert torch.equal(unpack_rows(xp.cpu(), cols)[:rows], xe.cpu())
    assert slot.tolist() == [-1 if i % 3 == 1 else 7 + i for i in range(rows)]
    assert qpos.tolist() == [-1 if i % 3 == 1 else 3 + i for i in range(rows)] and act.tolist() == [i % 3 != 1 for i in range(rows)]
    # norm of a sublayer's output, layer scale, residual sum, output norm; a plain part with a factor per row, and experts
    eps = 0.03  # (large enough to be seen)
    y, ys = pad(rnd(g, rows, width)).to(dtype), rnd(g, rows).abs()
    ex = pad(rnd(g, experts * rows, width)).to(dtype)
    idx, wt = torch.stack([torch.randperm(experts, generator=g)[:top] for _ in range(rows)]), torch.rand(rows, top, generator=g)
    coef, fcoef = pad(1 + 0.3 * rnd(g, 1, width))[0], pad(1 + 0.3 * rnd(g, 1, width))[0]
    for use in ("y", "y_scaled", "experts", "both"):
        x0 = pad(rnd(g, rows, width))
        want_y = torch.zeros(rows, cols, dtype=torch.float64)
        if use != "experts":
            want_y += y.double() * (1.0 if use == "y" else ys.double()[:, None])
        if use in ("experts", "both"):
            for r in range(rows):
                for e, w in zip(idx[r].tolist(), wt[r].double()):
                    want_y[r] += w * ex[e * rows + r].double()
        want = x0.double().clone()
        want[:, :width] = R.add_normed(x0.double()[:, :width], want_y[:, :width], coef.double()[:width] - 1.0, torch.ones(width, dtype=torch.float64), eps)
        xd, xe, xp = x0.to(dev), z(rows, cols), (z(32 * cols) if packed else None)
        nrm, nrmp = z(rows, cols), (z(32 * cols) if packed else None)
        experts_on = use in ("experts", "both")
        _call("residual_norm", xd, coef.to(dev), width, eps, y.to(dev) if use != "experts" else None,
              ys.to(dev) if use in ("y_scaled", "both") else None, ex.to(dev) if experts_on else None,
              idx.to(torch.int32).to(dev) if experts_on else None, wt.to(dev) if experts_on else None, xe, xp, fcoef.to(dev), nrm, nrmp, rows, 1, 1, cols, None, None, None)
        close(xd, want, torch.float32, f"residual {use}")
        assert torch.equal(xe, xd.to(dtype))
        wn = torch.zeros_like(want)
        wn[:, :width] = R.rms(want[:, :width], eps) * fcoef.double()[:width]
        close(nrm, wn, dtype, f"output norm {use}", tol=None if dtype == BF else 1e-5)
        if packed:
            assert torch.equal(unpack_rows(xp.cpu(), cols)[:rows], xe.cpu()) and torch.equal(unpack_rows(nrmp.cpu(), cols)[:rows], nrm.cpu())
    a = (2 * rnd(g, rows, 2 * cols)).to(dtype)
    close(_call("activate_rows", a.to(dev), 0, None, 0.0, 0.0), R.gelu_tanh(a.double()), dtype, "gelu")
    close(_call("activate_rows", a.to(dev), 1, None, 0.0, 0.0), R.silu(a.double()[:, :cols]) * a.double()[:, cols:], dtype, "silu * up")


def linear_batch_case(dev, rows, n, k, batch, seed=2):
    """Several products in one launch: a rows operand each or shared, results apart or side by side, only those selected."""
    from tah_amd import ops
    g = torch.Generator().manual_seed(seed)
    w, x = (rnd(g, batch, n, k) * k ** -0.5).to(BF), rnd(g, batch, rows, k).to(BF)
    wp = torch.cat([ops.linear_pack_weight(t.to(dev)) for t in w])
    xp = torch.cat([ops.linear_pack_rows(t.to(dev)) for t in x])
    want = torch.matmul(x.double(), w.double().transpose(1, 2))
    step = n + 8
    side = torch.zeros(32 * ((batch * step + 31) // 32 * 32), dtype=BF, device=dev)
    got = ops.linear_rows(wp, xp, rows, n, k, batch=batch, out_packed=side, packed_col_step=step)
    close(got.reshape(want.shape), want, BF, "batch")
    u = unpack_rows(side.cpu(), side.numel() // 32)
    for b in range(batch):
        assert torch.equal(u[:rows, b * step:b * step + n], got.reshape(want.shape)[b].cpu())
    close(ops.linear_rows(wp, xp[:32 * k].contiguous(), rows, n, k, batch=batch, shared_rows=True).reshape(want.shape),
          torch.matmul(x[:1].double(), w.double().transpose(1, 2)), BF, "shared rows")
    if batch > 2:
        out = torch.full((batch, rows, n), 5.0, dtype=BF, device=dev)
        ops.linear_rows(wp, xp, rows, n, k, batch=batch, out=out, select=i32([2, 0, 2], dev))
        assert torch.equal(out[0], got[0]) and torch.equal(out[2], got[2]) and bool((out[1] == 5.0).all())
    close(ops.linear_rows(ops.linear_pack_weight(w[0].to(dev)), xp[:32 * k].contiguous(), rows, n, k, gelu_tanh=True),
          R.gelu_tanh(want[0]), BF, "gelu tanh")


# ── gated delta rule ─────────────────────────────────────────────────────────────────────────────────────────────────
def delta_layer(dev, dtype, m, nslots, g, slow=True):
    """Weights with slow decay (tokens far back still matter) and the layer on poisoned slots."""
    from tah_amd import ops
    H, KH, D, V, taps = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
    nch = 2 * KH * D + H * V
    w = {"conv": rnd(g, nch, taps) * taps ** -0.5, "A_log": rnd(g, H) * 0.3 + (-5.0 if slow else 0.5), "dt_bias": rnd(g, H), "norm": 1 + 0.2 * rnd(g, V)}
    at, cols = (8 if D % 8 == 0 else 3), []   # (both the vector form and the element form of the kernels)
    for n in (KH * D, KH * D, H * V, H * V, H, H):  # q k v gate b a
        cols.append(at)
        at += n
    f = lambda t: t.float().to(dev)
    cs = torch.full((nslots, taps, nch), 7.0, dtype=dtype, device=dev)
    S = torch.full((nslots, H, D, V), -3.0, device=dev)
    at = (at + 7) // 8 * 8
    return ops.lib().DeltaLayer(f(w["conv"]), f(w["A_log"]), f(w["dt_bias"]), f(w["norm"]), cs, S, H, KH, D, V, cols, m["eps"]), w, cols, at, S


def delta_oracle(proj, w, m, cols):
    """[T, H * V] of one sequence from its projections (float64)."""
    H, KH, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    sizes = (KH * D, KH * D, H * V, H * V, H, H)
    q, k, v, gate, b, a = (proj[:, c:c + n] for c, n in zip(cols, sizes))
    cw, c0 = w["conv"].double(), KH * D
    q, k, v = R.short_conv(q, cw[:c0]), R.short_conv(k, cw[c0:2 * c0]), R.short_conv(v, cw[2 * c0:])
    T = proj.shape[0]
    q, k, v = R.unit(q.view(T, KH, D)) * D ** -0.5, R.unit(k.view(T, KH, D)), v.view(T, H, V)
    g = torch.exp(-torch.exp(w["A_log"].double()) * R.softplus(a + w["dt_bias"].double()))
    beta, outs, states = torch.sigmoid(b), [], []
    for i in range(H):
        j = i // (H // KH)
        o, S = R.delta_recurrence(q[:, j], k[:, j], v[:, i], g[:, i], beta[:, i])
        outs.append(R.rms(o, m["eps"]) * w["norm"].double() * R.silu(gate[:, i * V:(i + 1) * V]))
        states.append(S)
    return torch.cat(outs, -1), torch.stack(states)


def delta_case(dev, dtype, m, lens=(9, 4), cuts=((9,), (2, 2)), steps=3, seed=3):
    """Sequences run in portions, then token by token, on slots other sequences left; results and states against the oracle."""
    g = torch.Generator().manual_seed(seed)
    B = len(lens)
    layer, w, cols, width, S = delta_layer(dev, dtype, m, B + 2, g)
    HV = m["heads"] * m["vdim"]
    out_cols = (HV + 31) // 32 * 32
    slots = [B + 1 - b for b in range(B)]
    for rerun in range(2):  # the second time on slots the first sequences left
        proj = [(rnd(g, n + steps, width)).to(dtype) for n in lens]
        want, state = zip(*(delta_oracle(p.double(), w, m, cols) for p in proj))
        got = [[] for _ in lens]
        at = [0] * B
        for cut in range(max(len(c) for c in cuts)):
            live = [b for b in range(B) if cut < len(cuts[b])]
            ln = [cuts[b][cut] for b in live]
            rows = torch.cat([proj[b][at[b]:at[b] + n] for b, n in zip(live, ln)])
            P, cu = portions_of(ln, [at[b] for b in live], [slots[b] for b in live], dev)
            out = torch.full((rows.shape[0], out_cols), 9.0, dtype=dtype, device=dev)
            layer.portions(rows.to(dev), P, out)
            assert not out[:, HV:].any()
            for i, b in enumerate(live):
                got[b].append(out[cu[i]:cu[i + 1], :HV])
                at[b] += ln[i]
        for s in range(steps):
            rows = torch.stack([proj[b][lens[b] + s] for b in range(B)] + [proj[0][0]])  # and a row that is dropped
            out = torch.full((B + 1, out_cols), 9.0, dtype=dtype, device=dev)
            xp = torch.zeros(32 * out_cols, dtype=BF, device=dev) if dtype == BF else None
            layer.step(rows.to(dev), i32(slots + [-1], dev), i32([lens[b] + s for b in range(B)] + [4], dev), out, xp)
            assert not out[:, HV:].any() and not out[B].any()
            if xp is not None:
                assert torch.equal(unpack_rows(xp.cpu(), out_cols)[:B + 1], out.cpu())
            for b in range(B):
                got[b].append(out[b:b + 1, :HV])
        for b in range(B):
            close(torch.cat(got[b]), want[b], dtype, f"delta rule, sequence {b}")
            close(S[slots[b]], state[b], torch.float32, f"state of sequence {b}", tol=2e-5)
    assert bool((S[0] == -3.0).all())  # a slot nobody owned


# ── latent attention ─────────────────────────────────────────────────────────────────────────────────────────────────
def latent_case(dev, dtype, m, total, cuts, steps, capacity=None, slots=3, stand_out=True, seed=4):
    """One sequence next to a second, shorter one: portions of the given sizes, then single tokens, with its window inside
    a ring of ``capacity``.  With ``stand_out`` the scores of keys at distance window - 1 and window are raised far above
    the others, so that the key just inside decides a row's result and the one just outside would."""
    from tah_amd import ops
    from tah_amd.mixers import pad_to
    g = torch.Generator().manual_seed(seed)
    H, D, RD, V, C, W = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["mask"]["size"]
    Dp, Rp, Cp, Vp = pad_to(D), pad_to(RD), pad_to(C), pad_to(V, 16)
    cap = capacity or W
    ring = torch.full((slots, cap, Cp + Rp), 50.0, dtype=dtype, device=dev)
    layer = ops.lib().LatentLayer(ring, H, Dp, RD, Rp, C, Cp, Vp, W, m["scale"])
    eps = 1e-3
    norm = 1 + 0.2 * rnd(g, C)
    uk, uv = rnd(g, H, D, C) * C ** -0.5, rnd(g, H, V, C) * C ** -0.5
    uk, uv = uk.to(dtype), uv.to(dtype)
    half = RD // 2
    f = m["rot"]["base"] ** (-torch.arange(half, dtype=torch.float64) * 2 / RD)
    ang = torch.arange(total + steps + 8, dtype=torch.float64)[:, None] * f[None]
    cos, sin = ang.cos().float().to(dev), ang.sin().float().to(dev)
    ukp = torch.zeros(H, Dp, Cp, dtype=dtype); ukp[:, :D, :C] = uk
    uvp = torch.zeros(H, Vp, Cp, dtype=dtype); uvp[:, :V, :C] = uv
    other = max(2, total // 2)
    lens = [total, other]
    qs = [(rnd(g, n + steps, H, D + RD)).to(dtype) for n in lens]
    dkv = [(rnd(g, n + steps, C + RD)).to(dtype) for n in lens]
    if stand_out:  # queries of position p look for the latent of p - (W - 1) (visible) or, every other one, of p - W (not visible)
        c0, _ = R.latent_keys(dkv[0].double(), {"dkv": torch.eye(C + RD, dtype=torch.float64), "dkv.norm": norm.double()}, m, eps)
        for p in range(total + steps):
            j = p - (W - 1) - (p % 2)
            if j >= 0:
                k = torch.einsum("hdc,c->hd", uk.double(), c0[j])
                qs[0][p, :, :D] = (k / k.pow(2).sum(-1, keepdim=True) * (9.0 / m["scale"])).to(dtype)
    hq = Dp + Rp
    dcol = 8 + H * hq
    width = dcol + C + RD + 5
    projs = []
    for b in range(2):
        p = torch.zeros(lens[b] + steps, (width + 7) // 8 * 8, dtype=dtype)
        qv = p[:, 8:8 + H * hq].view(-1, H, hq)
        qv[:, :, :D], qv[:, :, Dp:Dp + RD] = qs[b][:, :, :D], qs[b][:, :, D:]
        p[:, dcol:dcol + C + RD] = dkv[b]
        projs.append(p)
    want = []
    for b in range(2):
        T = lens[b] + steps
        c, kr = R.latent_keys(dkv[b].double(), {"dkv": torch.eye(C + RD, dtype=torch.float64), "dkv.norm": norm.double()}, m, eps)
        ident = {"q": torch.eye(H * (D + RD), dtype=torch.float64), "uk": uk.double().reshape(H * D, C), "uv": uv.double().reshape(H * V, C),
                 "o": torch.eye(H * V, dtype=torch.float64)}
        want.append(R.latent_attention(qs[b].double().reshape(T, -1), ident, m, c, kr))
    owner = [2, 0]
    ws = torch.zeros(max(int(layer.decode_workspace(3)), 16), dtype=torch.uint8, device=dev)
    got, at = [[], []], [0, 0]
    second = [other - 2, 2] if other > 3 else [other]
    for i in range(max(len(cuts), len(second))):
        live = [b for b, c in ((0, cuts), (1, second)) if i < len(c)]
        ln = [(cuts, second)[b][i] for b in live]
        P, cu = portions_of(ln, [at[b] for b in live], [owner[b] for b in live], dev)
        proj = torch.cat([projs[b][at[b]:at[b] + n] for b, n in zip(live, ln)]).to(dev)
        pos = i32([p for b, n in zip(live, ln) for p in range(at[b], at[b] + n)], dev)
        new = torch.empty(cu[-1], Cp + Rp, dtype=dtype, device=dev)
        layer.prep(proj, 8, dcol, norm.to(dev), eps, cos, sin, pos, None, new, None, None)
        ck = [0]
        for b, n in zip(live, ln):
            ck.append(ck[-1] + n + min(at[b], cap - 1))
        ctx = torch.empty(ck[-1], Cp + Rp, dtype=dtype, device=dev)
        layer.context(P, i32(ck, dev), new, ctx)
        c = ctx[:, :Cp]
        k, v = (c @ ukp.view(-1, Cp).t().to(dev)), (c @ uvp.view(-1, Cp).t().to(dev))
        out = torch.full((cu[-1], H * Vp), 9.0, dtype=dtype, device=dev)
        layer.attend(P, i32(ck, dev), max(ln), proj, 8, k, v, ctx, out)
        for x, b in enumerate(live):
            got[b].append(out[cu[x]:cu[x + 1]].view(-1, H, Vp)[:, :, :V].reshape(ln[x], -1))
            at[b] += ln[x]
    for s in range(steps):
        proj = torch.stack([projs[0][total + s], projs[1][other + s], projs[0][0]]).to(dev)
        slot, pos = i32(owner + [-1], dev), i32([total + s, other + s, 3], dev)
        q_rows = torch.empty(H, 3, Dp, dtype=dtype, device=dev)
        qp = torch.zeros(H * 32 * Dp, dtype=BF, device=dev) if dtype == BF else None
        layer.prep(proj, 8, dcol, norm.to(dev), eps, cos, sin, pos, slot, None, qp, q_rows)
        if qp is not None:
            for h in range(H):
                assert torch.equal(unpack_rows(qp.view(H, -1)[h].cpu(), Dp)[:3], q_rows[h].cpu())
        q = torch.matmul(q_rows.float(), ukp.float().to(dev)).to(dtype).contiguous()
        o = torch.full((H, 3, Cp), 9.0, dtype=dtype, device=dev)
        op = torch.zeros(H * 32 * Cp, dtype=BF, device=dev) if dtype == BF else None
        layer.decode(slot, pos, q, proj, 8, op, o, ws)
        if op is not None:
            for h in range(H):
                assert torch.equal(unpack_rows(op.view(H, -1)[h].cpu(), Cp)[:3], o[h].cpu())
        assert not o[:, 2].any()
        y = torch.matmul(o.float(), uvp.float().transpose(1, 2).contiguous().to(dev))[:, :, :V]
        for b in range(2):
            got[b].append(y[:, b].reshape(1, -1).to(dtype))
    for b in range(2):
        # (scores of 9 and more: in bf16 the roundings of queries and keys move the weights by a few per cent)
        close(torch.cat(got[b]), want[b], dtype, f"latent attention, sequence {b}", tol=0.1 if dtype == BF else None)
    if stand_out:  # the window's edge is in the numbers: one position more or less is far outside the tolerance
        for wrong in (W - 1, W + 1):
            mm = dict(m, mask={"size": wrong})
            ident = {"q": torch.eye(H * (D + RD), dtype=torch.float64), "uk": uk.double().reshape(H * D, C),
                     "uv": uv.double().reshape(H * V, C), "o": torch.eye(H * V, dtype=torch.float64)}
            c, kr = R.latent_keys(dkv[0].double(), {"dkv": torch.eye(C + RD, dtype=torch.float64), "dkv.norm": norm.double()}, m, eps)
            bad = R.latent_attention(qs[0].double().reshape(total + steps, -1), ident, mm, c, kr)
            assert float((bad - want[0]).abs().max() / want[0].pow(2).mean().sqrt()) > 0.3
    assert bool((ring[1] == 50.0).all())  # a slot nobody owned


# ── mixture of experts ───────────────────────────────────────────────────────────────────────────────────────────────
def moe_case(dev, dtype, rows, width, ff, experts, top, shared_ff, seed=5):
    from tah_amd.mixers import MoeMlp, Router, Step, pad_to

    class Engine:
        packed = dtype == BF
        device = torch.device(dev)
    g = torch.Generator().manual_seed(seed)
    w = {"router": rnd(g, experts, width) * width ** -0.5 * 3, "gate": rnd(g, experts, ff, width) * width ** -0.5,
         "up": rnd(g, experts, ff, width) * width ** -0.5, "down": rnd(g, experts, width, ff) * ff ** -0.5}
    sh = None
    if shared_ff:
        sh = {"gate": rnd(g, shared_ff, width) * width ** -0.5, "up": rnd(g, shared_ff, width) * width ** -0.5,
              "down": rnd(g, width, shared_ff) * shared_ff ** -0.5, "sg": rnd(g, 1, width) * width ** -0.5 * 2}
    w = {k: t.to(dtype) for k, t in w.items()}
    sh = {k: t.to(dtype) for k, t in sh.items()} if sh else None
    cols = pad_to(width)
    x = rnd(g, rows, width).to(dtype).float()   # (a row and its element-type form agree: no close call between experts)
    xd = torch.nn.functional.pad(x, (0, cols - width)).to(dev)
    flat = {f"e{e}.{k}": w[k][e].double() for e in range(experts) for k in ("gate", "up", "down")}
    flat["router"] = w["router"].double()
    if sh:
        flat.update({"shared." + k: t.double() for k, t in sh.items()})
    want = R.moe_mlp(x.double(), flat, {"router": {"top": top}, "shared": sh})
    d = lambda t: {k: v.to(dev) for k, v in t.items()} if t else None
    b = MoeMlp(Router(top), d(w), d(sh), cols).bind(Engine)
    idx, _ = R.route(x.double(), w["router"].double(), top)
    pos = i32([0] * rows, dev)

    def total(r):
        y = torch.zeros(rows, cols, dtype=torch.float64)
        if r.y is not None:
            y += r.y.double().cpu() * (r.y_scale.double().cpu()[:, None] if r.y_scale is not None else 1.0)
        at = r.index.long().cpu() * r.index_scale + torch.arange(rows)[:, None] * r.index_row
        y += (r.experts.double().cpu()[at] * r.weight.double().cpu()[:, :, None]).sum(1)
        assert not y[:, width:].any()
        return y[:, :width]
    st = Step(xd, xd.to(dtype), pos, portions=object())
    r = b.portions(st)
    close(total(r), want, dtype, "experts, sorted rows")
    close(r.weight.sum(1), torch.ones(rows), torch.float32, "weights")
    index, _, _ = b._route(st)
    assert torch.equal(index.cpu().long().sort(1).values, idx.sort(1).values)
    if dtype == BF and rows <= 32:
        from tah_amd import ops
        st = Step(xd, xd.to(dtype), pos, ops.linear_pack_rows(xd.to(dtype)), slot=pos)
        close(total(b.rows(st)), want, dtype, "experts, decode rows")


# ── the whole decoder ────────────────────────────────────────────────────────────────────────────────────────────────
def delta_of(heads, kv, dim, vdim, conv):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv}}


def latent_of(heads, dim, rot, vdim, rank, window, base, scale, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "mask": {"size": window}, "rot": {"base": base, "dims": rot},
         "scale": scale}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m}


def dense_of(ff):
    return {"kind": "dense", "ff": ff}


def moe_of(experts, top, ff, shared):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}, "shared": {"ff": shared} if shared else None}


def config(width, vocab, layers, eps=1e-5):
    return {"architecture": "Zozosun", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": [dict(l, mlp=f) for l, f in layers]}


# sizes that are no multiples of anything, a source whose reader has the wider window, a layer without feed-forward, one
# key head, several, as many as heads, one tap, one expert per token, no shared expert
ODD = config(44, 61, [
    (latent_of(3, 20, 6, 12, 24, 5, 100.0, 0.3), moe_of(5, 1, 12, 0)),
    (delta_of(4, 1, 12, 20, 3), None),
    (latent_of(2, 8, 6, 28, 24, 11, 100.0, 0.5, kv_from=0), dense_of(52)),
    (delta_of(2, 2, 18, 7, 1), moe_of(3, 2, 20, 9)),
], eps=3e-3)
# multiples of the matrix steps, several heads per key head, two rings
EVEN = config(96, 128, [
    (delta_of(4, 2, 32, 64, 4), dense_of(160)),
    (latent_of(4, 64, 32, 64, 96, 9, 10000.0, 0.2), moe_of(8, 3, 32, 64)),
    (latent_of(20, 32, 16, 32, 64, 45, 1000.0, 0.6), dense_of(96)),
    (delta_of(2, 1, 64, 32, 2), moe_of(4, 4, 64, 32)),
    (latent_of(6, 32, 32, 16, 96, 30, 10000.0, 0.4, kv_from=1), None),
])
