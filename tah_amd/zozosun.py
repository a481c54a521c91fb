"""Zozosun: a decoder of gated delta-rule and sliding-window latent-attention layers, dense or mixture-of-experts
feed-forward, norms on the sublayers' outputs with a layer scale.  This module reads its configuration and tensor
names into the mechanisms of ``tah_amd.mixers``; everything that runs is there and in ``tah_amd.stack``.

Configuration: width, vocab, norm.eps, and layers, each with type ('delta' or 'latent_attention'), mixer and mlp:
  delta             heads, kv_heads, dim, vdim, conv (taps)
  latent_attention  heads, dim, rot_dim, vdim, kv_rank, scale, rot {base, dims}, mask {size}, optionally kv_from
  mlp               null, {kind: dense, ff}, or {kind: moe, router {experts, top}, expert {ff}, shared {ff} or null}
"""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

from ._capi import TahDuoError
from .mixers import DeltaMixer, DeltaSpec, DenseMlp, LatentAttention, LatentSpec, MoeMlp, Router, pad_to, padded
from .stack import StackEngine, StackLayer, StackModel, make_head, norm_coef

NAME = "Zozosun"


def mixer_spec(layer: dict, eps: float):
    m = layer["mixer"]
    if layer["type"] == "delta":
        if m["heads"] % m["kv_heads"]:
            raise TahDuoError("delta: heads must be a multiple of kv_heads")
        return DeltaSpec(m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"], eps)
    if layer["type"] == "latent_attention":
        rot, mask = m["rot"], m.get("mask") or {}
        if rot["dims"] != m["rot_dim"]:
            raise TahDuoError("latent_attention: rot.dims must be rot_dim")
        return LatentSpec(m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], float(rot["base"]), float(m["scale"]), eps,
                          mask.get("size"), m.get("kv_from"))
    raise TahDuoError(f"unknown layer type {layer['type']!r}")


def load(config: dict, tensors: Dict[str, torch.Tensor], device, dtype: torch.dtype = torch.bfloat16) -> StackModel:
    eps, width = float(config["norm"]["eps"]), config["width"]
    cols = pad_to(width)
    raw = lambda name: tensors[name].to(device)
    mat = lambda name: raw(name).to(dtype)

    def mixer(i: int, layer: dict):
        spec, pre = mixer_spec(layer, eps), f"l{i}.mix."
        if isinstance(spec, DeltaSpec):
            w = {k: mat(pre + k) for k in ("q", "k", "v", "g", "b", "a", "o")}
            w.update({f"conv_{k}": raw(f"{pre}{k}.conv") for k in "qkv"})
            w.update(a_log=raw(pre + "A_log"), dt_bias=raw(pre + "dt_bias"), norm=raw(pre + "norm"))
            return DeltaMixer(spec, w, cols)
        w = {k: mat(pre + k) for k in ("q", "uk", "uv", "o")}
        if spec.source is None:
            w.update(dkv=mat(pre + "dkv"), dkv_norm=raw(pre + "dkv.norm"))
        return LatentAttention(spec, w, cols)

    def mlp(i: int, spec: Optional[dict]):
        pre = f"l{i}.mlp."
        if not spec:
            return None
        if spec["kind"] == "dense":
            return DenseMlp({k: mat(pre + k) for k in ("up", "down")}, cols)
        if spec["kind"] != "moe":
            raise TahDuoError(f"unknown feed-forward {spec['kind']!r}")
        n, top = spec["router"]["experts"], spec["router"]["top"]
        w = {k: torch.stack([mat(f"{pre}e{e}.{k}") for e in range(n)]) for k in ("gate", "up", "down")}
        shared = {k: mat(f"{pre}shared.{k}") for k in ("gate", "up", "down", "sg")} if spec.get("shared") else None
        return MoeMlp(Router(top), dict(w, router=mat(pre + "router")), shared, cols)

    layers: List[StackLayer] = []
    for i, layer in enumerate(config["layers"]):
        ff = mlp(i, layer.get("mlp"))
        coef = lambda n: norm_coef(raw(f"l{i}.norm{n}"), raw(f"l{i}.ls{n}"), cols)
        layers.append(StackLayer(mixer(i, layer), coef(1), ff, coef(2) if ff is not None else None))
    return StackModel(width, config["vocab"], eps, padded(mat("embed"), config["vocab"], cols), make_head(mat("head"), cols),
                      norm_coef(raw("final.norm"), None, cols), layers)


def shapes(config: dict) -> Dict[str, tuple]:
    """Names and shapes of a model's tensors."""
    H = config["width"]
    out = {"embed": (config["vocab"], H)}
    for i, layer in enumerate(config["layers"]):
        s, p = mixer_spec(layer, float(config["norm"]["eps"])), f"l{i}."
        norms = ["1", "2"] if layer.get("mlp") else ["1"]
        out.update({f"{p}{k}{n}": (H,) for n in norms for k in ("norm", "ls")})
        p += "mix."
        if isinstance(s, DeltaSpec):
            for k, n in (("q", s.kv_heads * s.dim), ("k", s.kv_heads * s.dim), ("v", s.heads * s.vdim)):
                out[p + k], out[f"{p}{k}.conv"] = (n, H), (n, s.taps)
            out.update({p + "b": (s.heads, H), p + "a": (s.heads, H), p + "A_log": (s.heads,), p + "dt_bias": (s.heads,), p + "norm": (s.vdim,),
                        p + "g": (s.heads * s.vdim, H), p + "o": (H, s.heads * s.vdim)})
        else:
            out[p + "q"] = (s.heads * (s.dim + s.rot_dim), H)
            if s.source is None:
                out[p + "dkv"], out[p + "dkv.norm"] = (s.rank + s.rot_dim, H), (s.rank,)
            out.update({p + "uk": (s.heads * s.dim, s.rank), p + "uv": (s.heads * s.vdim, s.rank), p + "o": (H, s.heads * s.vdim)})
        p, f = f"l{i}.mlp.", layer.get("mlp")
        if not f:
            continue
        if f["kind"] == "dense":
            out[p + "up"], out[p + "down"] = (f["ff"], H), (H, f["ff"])
            continue
        for e in range(f["router"]["experts"]):
            out.update({f"{p}e{e}.gate": (f["expert"]["ff"], H), f"{p}e{e}.up": (f["expert"]["ff"], H), f"{p}e{e}.down": (H, f["expert"]["ff"])})
        out[p + "router"] = (f["router"]["experts"], H)
        if f.get("shared"):
            n = f["shared"]["ff"]
            out.update({p + "shared.gate": (n, H), p + "shared.up": (n, H), p + "shared.down": (H, n), p + "shared.sg": (1, H)})
    out["final.norm"], out["head"] = (H,), (config["vocab"], H)
    return out


def random_tensors(config: dict, device="cpu", seed: int = 0, dtype: torch.dtype = torch.bfloat16) -> Dict[str, torch.Tensor]:
    """Random weights of a model's shapes (benchmarks and tests)."""
    g = torch.Generator(device=device).manual_seed(seed)
    r = lambda *s: torch.randn(*s, generator=g, device=device)
    out = {}
    for name, s in shapes(config).items():
        leaf = name.rsplit(".", 1)[-1]
        if leaf == "A_log":
            t = torch.rand(*s, generator=g, device=device) * 2.0 - 3.0
        elif leaf.startswith("ls"):
            t = 0.5 + 0.2 * r(*s)
        elif name.endswith("dkv.norm") or name.endswith("mix.norm"):
            t = 1.0 + 0.1 * r(*s)
        elif len(s) == 1:
            t = 0.1 * r(*s)
        elif leaf == "conv":
            t = r(*s) * s[1] ** -0.5
        else:
            t = r(*s) * (1.0 if name == "embed" else s[1] ** -0.5)
        out[name] = t.to(dtype)
    return out


def engine(model: StackModel, batch: int, max_len: int, *, device="cuda", **kw) -> StackEngine:
    return StackEngine(model, batch, max_len, device=device, **kw)
