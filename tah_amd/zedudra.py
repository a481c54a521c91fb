"""Zedudra: a decoder of sliding-window attention layers that keep a sequence's first tokens and whose keys are their values,
with a short convolution of the mixer's input, dense or mixture-of-experts feed-forward, norms over groups of columns in
front of and behind every sublayer, and layers that may run on another layer's weights.  This module reads its configuration
and tensor names into the mechanisms of ``tah_amd.mixers``; everything that runs is there and in ``tah_amd.stack``.

Configuration: width, vocab, embedding.scale, norm {eps, groups}, canon {taps}, and layers, each with type 'attention', mixer,
mlp and optionally weights_of (the layer whose tensors it uses):
  mixer  heads, kv_heads, dim, vdim, scale, rot {base, dims}, mask {size, keep_first}
  mlp    null, {kind: dense, ff}, or {kind: moe, router {experts, top, groups {count, keep}}, expert {ff, limit}}
"""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

from ._capi import TahDuoError
from .mixers import DenseMlp, MoeMlp, Router, WindowAttention, WindowSpec, clamped_gate, padded, xielu
from .stack import Columns, StackEngine, StackLayer, StackModel, make_head, norm_coef

NAME = "Zedudra"


def mixer_spec(layer: dict) -> WindowSpec:
    if layer["type"] != "attention":
        raise TahDuoError(f"unknown layer type {layer['type']!r}")
    m = layer["mixer"]
    rot, mask = m.get("rot") or {"base": 1.0, "dims": 0}, m.get("mask") or {}
    return WindowSpec(m["heads"], m["kv_heads"], m["dim"], m["vdim"], rot["dims"], float(rot["base"]), float(m["scale"]), mask.get("size"),
                      mask.get("keep_first") or 0)


def router(spec: dict) -> Router:
    groups = spec.get("groups") or {"count": 1, "keep": 1}
    return Router(spec["top"], True, groups["count"], groups["keep"])


def owner(config: dict, i: int) -> int:
    """The layer whose tensors layer i uses."""
    seen = set()
    while config["layers"][i].get("weights_of") is not None:
        if i in seen:
            raise TahDuoError("layers that use each other's weights in a circle")
        seen.add(i)
        i = config["layers"][i]["weights_of"]
        if not 0 <= i < len(config["layers"]):
            raise TahDuoError(f"weights of layer {i}, which does not exist")
    return i


def load(config: dict, tensors: Dict[str, torch.Tensor], device, dtype: torch.dtype = torch.bfloat16) -> StackModel:
    eps, at = float(config["norm"]["eps"]), Columns(config["width"], config["norm"]["groups"])
    cols = at.cols
    raw = lambda name: tensors[name].to(device)
    mat = lambda name: raw(name).to(dtype)
    reads = lambda name: at.spread(mat(name), 1)    # a weight that is applied to a row of the model's width ...
    writes = lambda name: at.spread(mat(name), 0)   # ... and one that makes one
    coef = lambda name: norm_coef(at.spread(raw(name)), None, cols, zero_centred=False)

    def mlp(pre: str, spec: Optional[dict]):
        if not spec:
            return None
        if spec["kind"] == "dense":
            return DenseMlp({"up": reads(pre + "up"), "down": writes(pre + "down")}, cols, xielu(*raw(pre + "act").double().tolist()))
        if spec["kind"] != "moe":
            raise TahDuoError(f"unknown feed-forward {spec['kind']!r}")
        each = lambda f, leaf: torch.stack([f(f"{pre}e{e}.{leaf}") for e in range(spec["router"]["experts"])])
        w = {"router": reads(pre + "router"), "gate": each(reads, "gate"), "up": each(reads, "up"), "down": each(writes, "down")}
        return MoeMlp(router(spec["router"]), w, None, cols, clamped_gate(float(spec["expert"]["limit"])))

    def layer_of(i: int) -> StackLayer:
        layer, p = config["layers"][i], f"l{i}."
        w = {k: reads(f"{p}mix.{k}") for k in ("q", "k", "g")}
        taps = at.spread(raw(p + "canon1").float(), 0)
        if taps.shape[1] != config["canon"]["taps"]:
            raise TahDuoError(f"{p}canon1 has {taps.shape[1]} taps, the configuration says {config['canon']['taps']}")
        ff = mlp(p + "mlp.", layer.get("mlp"))
        return StackLayer(WindowAttention(mixer_spec(layer), dict(w, o=writes(p + "mix.o")), cols), coef(p + "norm1b"), ff,
                          coef(p + "norm2b") if ff is not None else None, coef(p + "norm1"), coef(p + "norm2") if ff is not None else None,
                          padded(taps.t(), taps.shape[1], cols))

    made: Dict[int, StackLayer] = {}
    layers: List[StackLayer] = []
    for i in range(len(config["layers"])):
        j = owner(config, i)
        if j not in made:
            made[j] = layer_of(j)
        layers.append(made[j])
    return StackModel(config["width"], config["vocab"], eps, padded(reads("embed"), config["vocab"], cols), make_head(reads("head"), cols),
                      coef("final.norm"), layers, at.groups, float(config["embedding"]["scale"]))


def shapes(config: dict) -> Dict[str, tuple]:
    """Names and shapes of a model's tensors."""
    H = config["width"]
    out = {"embed": (config["vocab"], H)}
    for i, layer in enumerate(config["layers"]):
        if owner(config, i) != i:
            continue
        s, p, f = mixer_spec(layer), f"l{i}.", layer.get("mlp")
        out.update({p + n: (H,) for n in (("norm1", "norm1b", "norm2", "norm2b") if f else ("norm1", "norm1b"))})
        out.update({p + "canon1": (H, config["canon"]["taps"]), p + "mix.q": (s.heads * s.dim, H), p + "mix.k": (s.kv_heads * s.dim, H),
                    p + "mix.g": (s.heads, H), p + "mix.o": (H, s.heads * s.vdim)})
        p += "mlp."
        if not f:
            continue
        if f["kind"] == "dense":
            out.update({p + "up": (f["ff"], H), p + "down": (H, f["ff"]), p + "act": (2,)})
            continue
        n = f["expert"]["ff"]
        for e in range(f["router"]["experts"]):
            out.update({f"{p}e{e}.gate": (n, H), f"{p}e{e}.up": (n, H), f"{p}e{e}.down": (H, n)})
        out[p + "router"] = (f["router"]["experts"], H)
    out["final.norm"], out["head"] = (H,), (config["vocab"], H)
    return out


def random_tensors(config: dict, device="cpu", seed: int = 0, dtype: torch.dtype = torch.bfloat16) -> Dict[str, torch.Tensor]:
    """Random weights of a model's shapes (benchmarks and tests)."""
    g = torch.Generator(device=device).manual_seed(seed)
    r = lambda *s: torch.randn(*s, generator=g, device=device)
    out = {}
    for name, s in shapes(config).items():
        leaf = name.rsplit(".", 1)[-1]
        if leaf.startswith("norm"):
            t = 1.0 + 0.1 * r(*s)
        elif leaf == "act":
            t = 0.5 * r(*s)
        elif leaf == "canon1":
            t = 0.5 * r(*s) * s[1] ** -0.5
        else:
            t = r(*s) * s[1] ** -0.5
        out[name] = t.to(dtype)
    return out


def engine(model: StackModel, batch: int, max_len: int, *, device="cuda", **kw) -> StackEngine:
    return StackEngine(model, batch, max_len, device=device, **kw)
