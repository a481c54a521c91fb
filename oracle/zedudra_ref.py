"""Plain, slow implementation of the Zedudra decoder (test oracle): one function per mechanism, one token or one head at a
time where that is the shortest way to say it, in the dtype of the tensors it gets (float64 in the tests).  It shares no
code with the package.

A model is a configuration dict (the parsed config.json) and a dict of tensors.  ``forward`` runs one whole sequence;
nothing here knows about caches, portions or batches.
"""
from __future__ import annotations

import math

import torch


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def softplus(x):
    return torch.log1p(torch.exp(-x.abs())) + x.clamp_min(0)


def group_norm(x, w, groups, eps):
    """Every group of consecutive entries divided by its own root mean square, then the weight."""
    size = x.shape[-1] // groups
    out = []
    for g in range(groups):
        part = x[..., g * size:(g + 1) * size]
        out.append(part / torch.sqrt((part * part).mean(-1, keepdim=True) + eps))
    return torch.cat(out, -1) * w


def add_conv(h, w):
    """h [T, channels] plus a causal convolution of it; w [channels, taps], last column for the current token."""
    T, taps = h.shape[0], w.shape[1]
    y = h.clone()
    for j in range(taps):
        back = taps - 1 - j
        if back < T:
            y[back:] += w[:, j] * h[:T - back]
    return y


def rotate_pairs(x, pos, base, dims):
    """x [T, ..., D]: entries 2 i and 2 i + 1, i < dims / 2, turned by pos * base^(-2 i / dims)."""
    y = x.clone()
    for i in range(dims // 2):
        a = pos.double() * base ** (-2.0 * i / dims)
        while a.dim() < x.dim() - 1:
            a = a.unsqueeze(-1)
        c, s = torch.cos(a).to(x.dtype), torch.sin(a).to(x.dtype)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        y[..., 2 * i], y[..., 2 * i + 1] = u * c - v * s, v * c + u * s
    return y


def visible(i, j, size, keep):
    return (j <= i) & ((i - j < size) | (j < keep))


def attention(q, k, v, m):
    """q [T, heads, dim], k [T, kv_heads, dim], v [T, kv_heads, vdim] (unrotated) -> [T, heads, vdim]."""
    T, H, per = q.shape[0], q.shape[1], q.shape[1] // k.shape[1]
    pos = torch.arange(T)
    qr, kr = (rotate_pairs(x, pos, m["rot"]["base"], m["rot"]["dims"]) for x in (q, k))
    seen = visible(pos[:, None], pos[None], m["mask"]["size"], m["mask"]["keep_first"])
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for h in range(H):
        s = (qr[:, h] @ kr[:, h // per].t()) * m["scale"]
        out[:, h] = torch.softmax(s.masked_fill(~seen, -math.inf), -1) @ v[:, h // per]
    return out


def attention_mixer(h, w, m):
    """Keys are values; one gate per head."""
    T, H, G, D = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q, k = (h @ w["q"].t()).view(T, H, D), (h @ w["k"].t()).view(T, G, D)
    out = attention(q, k, k, m) * sigmoid(h @ w["g"].t())[:, :, None]
    return out.reshape(T, -1) @ w["o"].t()


def xielu(z, p, q):
    return torch.where(z > 0, softplus(p) * z * z, (0.5 + softplus(q)) * (torch.exp(z.clamp_max(0)) - 1 - z)) + z / 2


def dense_mlp(h, w):
    return xielu(h @ w["up"].t(), w["act"][0], w["act"][1]) @ w["down"].t()


def clamped_gate(g, u, limit):
    g, u = g.clamp(max=limit), u.clamp(-limit, limit)
    return g * sigmoid(1.702 * g) * (u + 1)


def expert(h, w, limit):
    return clamped_gate(h @ w["gate"].t(), h @ w["up"].t(), limit) @ w["down"].t()


def route(h, w_router, top, groups):
    """Chosen experts and their weights per token: sigmoid scores, the best groups by their two largest, the largest
    in those."""
    scores = sigmoid(h @ w_router.t())
    idx = []
    for s in scores.tolist():
        n, size = groups["count"], len(s) // groups["count"]
        best = sorted(range(n), key=lambda g: -sum(sorted(s[g * size:(g + 1) * size])[-2:]))
        allowed = [e for g in best[:groups["keep"]] for e in range(g * size, (g + 1) * size)]
        idx.append(sorted(allowed, key=lambda e: -s[e])[:top])
    idx = torch.tensor(idx)
    return idx, scores.gather(1, idx)


def moe_mlp(h, w, spec):
    idx, p = route(h, w["router"], spec["router"]["top"], spec["router"]["groups"])
    out = torch.zeros_like(h)
    for e in range(spec["router"]["experts"]):
        y = expert(h, part(w, f"e{e}."), spec["expert"]["limit"])
        for c in range(idx.shape[1]):
            out += torch.where(idx[:, c:c + 1] == e, p[:, c:c + 1] * y, torch.zeros_like(y))
    return out


def part(w, prefix):
    return {k[len(prefix):]: t for k, t in w.items() if k.startswith(prefix)}


def forward(cfg, tensors, tokens, trace=None):
    """Logits [T, vocab] of one sequence.  ``trace``: list that receives the residual stream after every layer."""
    norm = lambda x, w: group_norm(x, w, cfg["norm"]["groups"], cfg["norm"]["eps"])
    x = tensors["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
    for i, layer in enumerate(cfg["layers"]):
        L = part(tensors, f"l{layer.get('weights_of', i)}.")
        h = add_conv(norm(x, L["norm1"]), L["canon1"])
        x = x + norm(attention_mixer(h, part(L, "mix."), layer["mixer"]), L["norm1b"])
        if layer.get("mlp"):
            h, w = norm(x, L["norm2"]), part(L, "mlp.")
            x = x + norm(dense_mlp(h, w) if layer["mlp"]["kind"] == "dense" else moe_mlp(h, w, layer["mlp"]), L["norm2b"])
        if trace is not None:
            trace.append(x.clone())
    return norm(x, tensors["final.norm"]) @ tensors["head"].t()
