"""Whole decoders on the layer-by-layer engine, any design of the registry, against the design's plain oracle in float64."""
from __future__ import annotations

import copy
import importlib

import torch

from tests import zedudra_cases, zozosun_cases
from tests.zozosun_cases import BF, DTYPES  # noqa: F401

CONFIGS = {"zozosun odd": zozosun_cases.ODD, "zozosun even": zozosun_cases.EVEN,
           "zedudra odd": zedudra_cases.ODD, "zedudra even": zedudra_cases.EVEN, "zedudra plain": zedudra_cases.PLAIN}


def design(cfg):
    """The package's module of a configuration's design."""
    return importlib.import_module("tah_amd." + cfg["architecture"].lower())


def oracle(cfg):
    return importlib.import_module(f"oracle.{cfg['architecture'].lower()}_ref")


def without_close_calls(cfg):
    """The same model with every expert chosen for every token: between bf16 and float64 a choice of experts can flip, and a
    flipped choice is no fault.  (What choosing does is checked in float32, and in bf16 with the mechanism alone.)"""
    c = copy.deepcopy(cfg)
    for layer in c["layers"]:
        if layer["mlp"] and layer["mlp"]["kind"] == "moe":
            r = layer["mlp"]["router"]
            r["top"] = r["experts"]
            if r.get("groups"):
                r["groups"]["keep"] = r["groups"]["count"]
    return c


def tensors_for(cfg, seed=0, sharp=2.0):
    """Random weights with peaked attention (a key more or less shows) and slow decay (a lost state shows)."""
    t = design(cfg).random_tensors(cfg, seed=seed)
    for name, v in t.items():
        if name.endswith("A_log"):
            t[name] = v - 2.0
        i = int(name[1:name.index(".")]) if name[0] == "l" else None
        if i is not None and cfg["layers"][i]["type"].endswith("attention") and name == f"l{i}.mix.q":
            t[name] = (v.float() * sharp).to(BF)
    return t


def oracle_logits(cfg, tensors, tokens):
    return oracle(cfg).forward(cfg, {k: v.double() for k, v in tensors.items()}, tokens)


class Check:
    """Logits of the engine against the oracle's: root mean square of the difference relative to the oracle's own, per
    position.  bf16 differs by its roundings, which a sequence of random layers amplifies.  In float32 a position where the
    model itself magnifies roundings (a group of columns that nearly cancels in front of its norm) may differ by eight
    times what relative changes of 2^-24 in the weights make of it."""
    LIMIT = {torch.float32: 2e-5, BF: 0.1}

    def __init__(self, cfg, tensors, dtype):
        self.cfg, self.t, self.dtype, self.memo = cfg, tensors, dtype, {}

    def want(self, tokens):
        key = tuple(tokens)
        if key not in self.memo:
            self.memo[key] = oracle_logits(self.cfg, self.t, list(tokens))
        return self.memo[key]

    def __call__(self, got, tokens, places, what):
        w = self.want(tokens)[list(places)]
        d = got.double().cpu() - w
        err = (d.pow(2).mean(-1).sqrt() / w.pow(2).mean(-1).sqrt())
        limit = torch.full_like(err, self.LIMIT[self.dtype])
        if self.dtype == torch.float32 and float(err.max()) > self.LIMIT[self.dtype]:
            limit = torch.maximum(limit, 8.0 * self.sensitivity(tokens)[list(places)])
        bad = int((err / limit).argmax())
        assert bool((err <= limit).all()), f"{what}: position {list(places)[bad]} differs by {float(err[bad]):.2e}"
        return float(err.max())

    def sensitivity(self, tokens, runs=12):
        w, out = self.want(tokens), []
        for i in range(runs):
            g = torch.Generator().manual_seed(i)
            moved = {k: v.double() * (1 + torch.randn(v.shape, generator=g, dtype=torch.float64) * 2.0 ** -24) for k, v in self.t.items()}
            out.append((oracle(self.cfg).forward(self.cfg, moved, list(tokens)) - w).pow(2).mean(-1).sqrt() / w.pow(2).mean(-1).sqrt())
        return torch.stack(out).max(0).values


def load(cfg, tensors, dtype, dev):
    return design(cfg).load(cfg, {k: v.to(dev) for k, v in tensors.items()}, dev, dtype)


def tokens_of(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def run_cut(eng, check, tokens, cuts, what, slot=None):
    """One sequence in portions of the given sizes (the rest token by token), every position's logits checked."""
    s = eng.alloc() if slot is None else slot
    at, worst = 0, 0.0
    cuts = list(cuts) + [1] * (len(tokens) - sum(cuts))
    for n in cuts:
        lg = eng.extend([(s, tokens[at:at + n])])
        worst = max(worst, check(lg, tokens, range(at, at + n), f"{what} {cuts[:6]}... portion at {at}"))
        at += n
    if slot is None:
        eng.release(s)
    return worst


def wrong_oracles_differ(cfg, tensors, tokens):
    """The weights of these tests let faults show: an oracle with a window or its kept tokens off by one or a lost state is
    much further away than the float32 tolerance, at some position."""
    good = oracle_logits(cfg, tensors, tokens)
    lim = 0.05

    def far(cfg2=cfg, t2=tensors, cut=0):
        bad = oracle_logits(cfg2, t2, tokens[cut:])
        d = (bad - good[cut:]).pow(2).mean(-1).sqrt() / good[cut:].pow(2).mean(-1).sqrt()
        return float(d[-8:].max() if cut else d.max())
    for i, layer in enumerate(cfg["layers"]):
        mask = layer["mixer"].get("mask") or {}
        for key in ("size", "keep_first"):
            for delta in (-1, 1):
                if key not in mask or mask[key] + delta < (key == "size"):
                    continue
                c = copy.deepcopy(cfg)
                c["layers"][i]["mixer"]["mask"][key] += delta
                assert far(c) > lim, f"mask.{key} off by {delta} in layer {i} does not show"
    assert far(cut=len(tokens) // 2) > lim, "a lost state does not show"
