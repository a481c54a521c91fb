"""Plain, slow implementation of the Zozosun decoder (test oracle): one function per mechanism, one token or one head
at a time where that is the shortest way to say it, in the dtype of the tensors it gets (float64 in the tests).  It
shares no code with the package.

A model is a configuration dict (the parsed config.json) and a dict of tensors.  ``forward`` runs one whole sequence;
nothing here knows about caches, portions or batches.
"""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(x):
    return x * torch.sigmoid(x)


def gelu_tanh(x):
    return 0.5 * x * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (x + 0.044715 * x ** 3)))


def softplus(x):
    return torch.where(x > 0, x, torch.zeros_like(x)) + torch.log1p(torch.exp(-x.abs()))


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def short_conv(x, w):
    """x [T, channels], w [channels, taps], last column for the current token; zeros before the start; then silu."""
    T, taps = x.shape[0], w.shape[1]
    y = torch.zeros_like(x)
    for t in range(T):
        for j in range(taps):
            s = t - (taps - 1 - j)
            if s >= 0:
                y[t] += w[:, j] * x[s]
    return silu(y)


def delta_recurrence(q, k, v, g, beta, state=None):
    """One head.  q, k [T, dim], v [T, vdim], decay g and step beta [T].  Returns the read-outs [T, vdim] and the state
    [dim, vdim] after the last token."""
    S = torch.zeros(q.shape[1], v.shape[1], dtype=q.dtype) if state is None else state.clone()
    out = torch.zeros(q.shape[0], v.shape[1], dtype=q.dtype)
    for t in range(q.shape[0]):
        S = g[t] * S
        u = beta[t] * (v[t] - S.t() @ k[t])
        S = S + torch.outer(k[t], u)
        out[t] = S.t() @ q[t]
    return out, S


def delta_mixer(h, w, m, eps):
    """h [T, width]; w: tensor by short name ('q', 'q.conv', ...); m: the mixer's sizes."""
    T = h.shape[0]
    H, KH, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = short_conv(h @ w["q"].t(), w["q.conv"]).view(T, KH, D)
    k = short_conv(h @ w["k"].t(), w["k.conv"]).view(T, KH, D)
    v = short_conv(h @ w["v"].t(), w["v.conv"]).view(T, H, V)
    q, k = unit(q) * D ** -0.5, unit(k)
    beta = torch.sigmoid(h @ w["b"].t())
    g = torch.exp(-torch.exp(w["A_log"]) * softplus(h @ w["a"].t() + w["dt_bias"]))
    gate = silu(h @ w["g"].t()).view(T, H, V)
    outs = []
    for i in range(H):
        j = i // (H // KH)
        o, _ = delta_recurrence(q[:, j], k[:, j], v[:, i], g[:, i], beta[:, i])
        outs.append(rms(o, eps) * w["norm"] * gate[:, i])
    return torch.cat(outs, -1) @ w["o"].t()


def rotate(x, pos, base, dims):
    """Rotary positions on the last axis's first ``dims`` entries, entry i paired with i + dims / 2."""
    half = dims // 2
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(half)], dtype=torch.float64)
    a = (pos.double()[:, None] * f[None]).to(x.dtype)
    while a.dim() < x.dim():
        a = a.unsqueeze(1)
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * a.cos() - v * a.sin(), v * a.cos() + u * a.sin(), x[..., dims:]], -1)


def latent_keys(h, w, m, eps):
    """The latent c [T, kv_rank] and the rotated key part [T, rot_dim]."""
    dkv = h @ w["dkv"].t()
    c = rms(dkv[:, :m["kv_rank"]], eps) * w["dkv.norm"]
    return c, rotate(dkv[:, m["kv_rank"]:], torch.arange(h.shape[0]), m["rot"]["base"], m["rot"]["dims"])


def visible(i, j, window):
    return 0 <= i - j < window


def latent_attention(h, w, m, c, kr):
    T, H, D, R, V = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    q = (h @ w["q"].t()).view(T, H, D + R)
    qr = rotate(q[..., D:], torch.arange(T), m["rot"]["base"], m["rot"]["dims"])
    kn = (c @ w["uk"].t()).view(T, H, D)
    v = (c @ w["uv"].t()).view(T, H, V)
    mask = torch.tensor([[visible(i, j, m["mask"]["size"]) for j in range(T)] for i in range(T)])
    out = torch.zeros(T, H, V, dtype=h.dtype)
    for n in range(H):
        s = (q[:, n, :D] @ kn[:, n].t() + qr[:, n] @ kr.t()) * m["scale"]
        p = torch.softmax(s.masked_fill(~mask, -math.inf), -1)
        out[:, n] = p @ v[:, n]
    return out.reshape(T, H * V) @ w["o"].t()


def dense_mlp(h, w):
    return gelu_tanh(h @ w["up"].t()) @ w["down"].t()


def gated_mlp(h, w):
    return (silu(h @ w["gate"].t()) * (h @ w["up"].t())) @ w["down"].t()


def route(h, w_router, top):
    """Chosen experts and their weights per token."""
    z = h @ w_router.t()
    vals, idx = torch.topk(z, top, dim=-1)
    return idx, torch.softmax(vals, -1)


def moe_mlp(h, w, spec):
    idx, p = route(h, w["router"], spec["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, pe in zip(idx[t].tolist(), p[t]):
            out[t] += pe * gated_mlp(h[t], part(w, f"e{e}."))
    if spec.get("shared"):
        s = part(w, "shared.")
        out += torch.sigmoid(h @ s["sg"].t()) * gated_mlp(h, s)
    return out


def part(w, prefix):
    return {k[len(prefix):]: t for k, t in w.items() if k.startswith(prefix)}


def add_normed(x, y, norm, scale, eps):
    """Norm on a sublayer's output (weight around zero), layer scale, residual."""
    return x + rms(y, eps) * (1.0 + norm) * scale


def forward(cfg, tensors, tokens, trace=None):
    """Logits [T, vocab] of one sequence.  ``trace``: list that receives the residual stream after every layer."""
    eps = cfg["norm"]["eps"]
    x = tensors["embed"][torch.as_tensor(tokens)]
    latents = {}
    for i, layer in enumerate(cfg["layers"]):
        L = part(tensors, f"l{i}.")
        w, m = part(L, "mix."), layer["mixer"]
        if layer["type"] == "delta":
            y = delta_mixer(x, w, m, eps)
        else:
            if "kv_from" in m:
                c, kr = latents[m["kv_from"]]
            else:
                c, kr = latents[i] = latent_keys(x, w, m, eps)
            y = latent_attention(x, w, m, c, kr)
        x = add_normed(x, y, L["norm1"], L["ls1"], eps)
        if layer.get("mlp"):
            mw = part(L, "mlp.")
            y = dense_mlp(x, mw) if layer["mlp"]["kind"] == "dense" else moe_mlp(x, mw, layer["mlp"])
            x = add_normed(x, y, L["norm2"], L["ls2"], eps)
        if trace is not None:
            trace.append(x.clone())
    return rms(x, eps) * (1.0 + tensors["final.norm"]) @ tensors["head"].t()
