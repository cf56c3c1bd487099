"""Tiny Vufizen configurations that differ in every size and option, and random weights for them.

The tensor list is written out here from the design (not asked of the package), so a part that expects another name or
shape fails to load.  Weights are drawn so that the mechanisms matter: matrices N(0, 1/in), the maps' lambda away from
`diff`, convolution taps of one size, gates whose channels remember from a few tokens to hundreds, floors from 0 to
close to 1, a norm's single number away from 1.  `sharpened` multiplies every attention's `scale` so that a query
singles out a few keys, and a key that is lost or read from a wrong page changes the logits by far more than rounding."""
from __future__ import annotations

import copy
import json
import os
from typing import Dict

import torch


def attn(heads, kv_heads, dim, vdim, scale, conv=4, diff=0.5, base=10000.0, turned=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "conv": conv, "diff": diff}
    turned = dim if turned is None else turned
    if turned:
        m["rot"] = {"base": base, "dims": turned}
    return {"type": "attention", "mixer": m}


def hgrn2(heads, dim, vdim):
    return {"type": "hgrn2", "mixer": {"heads": heads, "dim": dim, "vdim": vdim}}


def moe(experts, top, ff, shared=None):
    f = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}
    if shared is not None:
        f["shared"] = {"ff": shared}
    return f


def layer(mixer, mlp):
    return {**mixer, "mlp": mlp}


def model(vocab, width, layers, eps=1e-6):
    return {"architecture": "Vufizen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


def again(layers, i):
    """Layer i once more, with its tensors."""
    return {**copy.deepcopy(layers[i]), "weights_of": i}


# A: both mixers in turn, grouped keys with values wider than a map, part of a map turning, a convolution of four taps,
# routed experts with and without a shared one, a layer without feed-forward, three layers that run again (one of them a
# second time, through a layer that has no tensors either).
_A = [layer(attn(4, 2, 8, 12, 0.4, conv=4, diff=0.3, base=500.0, turned=6), moe(5, 2, 24, shared=16)),
      layer(hgrn2(3, 12, 10), moe(4, 3, 16)),
      layer(attn(2, 1, 12, 8, 0.3, conv=2, diff=0.8, base=50000.0), None)]
CFG_A = model(211, 48, _A + [again(_A, 1), again(_A, 0)], eps=1e-5)
CFG_A["layers"].append({**copy.deepcopy(CFG_A["layers"][3]), "weights_of": 3})
# B: every count 1 and every size equal where the design lets them differ: one head, one map's size for keys, values and
# state, one tap, one expert, nothing turning, nothing taken off ahead of the learned part (diff 0).
CFG_B = model(97, 64, [layer(attn(1, 1, 64, 64, 0.125, conv=1, diff=0.0, turned=0), moe(1, 1, 64, shared=64)),
                       layer(hgrn2(1, 64, 64), moe(1, 1, 64))])
# C: sizes that fit no vector width: a width of 50, maps of 11, values of 13, a state of 10 x 7, three taps, feed-forwards of
# 30 and 22.
CFG_C = model(101, 50, [layer(attn(3, 3, 11, 13, 0.5, conv=3, diff=0.2, base=777.0, turned=10), moe(3, 2, 30, shared=22)),
                        layer(hgrn2(5, 10, 7), moe(3, 3, 30)),
                        layer(hgrn2(2, 21, 33), None)], eps=1e-5)
# D: the matrix cores' sizes with long sequences: maps of 64 (keys of 128) with values of 128 and of 64, a state of 128 x 128,
# one of 48 x 160, a convolution of six taps.
_D = [layer(attn(4, 1, 64, 128, 0.15, conv=4, diff=0.5, base=30000.0, turned=32), moe(6, 2, 32, shared=16)),
      layer(hgrn2(2, 128, 128), moe(4, 1, 64)),
      layer(attn(4, 2, 64, 64, 0.15, conv=6, diff=0.6, base=1000.0), None),
      layer(hgrn2(2, 48, 160), moe(6, 2, 32))]
CFG_D = model(150, 128, _D + [again(_D, 0), again(_D, 3)])
# E: keys too wide for the chunks (the recurrence walks a prompt), keys of 48 on the matrix cores, a state with columns but
# one row.
CFG_E = model(83, 40, [layer(hgrn2(2, 150, 20), moe(3, 1, 16)),
                       layer(attn(2, 2, 24, 48, 0.3, conv=5, diff=0.4, base=100.0, turned=8), moe(3, 2, 24, shared=8)),
                       layer(hgrn2(4, 1, 24), moe(2, 2, 8))])
CONFIGS = {"A": CFG_A, "B": CFG_B, "C": CFG_C, "D": CFG_D, "E": CFG_E}


def sharpened(cfg: dict, factor: float) -> dict:
    """The same model with every attention's `scale` multiplied: its queries single out few of the keys they see."""
    out = copy.deepcopy(cfg)
    for L in out["layers"]:
        if L["type"] == "attention":
            L["mixer"]["scale"] = L["mixer"]["scale"] * factor
    return out


def tensor_shapes(cfg: dict) -> Dict[str, tuple]:
    """Every tensor of a model, from the design."""
    W, V = cfg["width"], cfg["vocab"]
    out = {"embed": (V, W), "final.norm": (), "head": (V, W)}
    for i, L in enumerate(cfg["layers"]):
        if L.get("weights_of") is not None:
            continue
        p, m, f = f"l{i}.", L["mixer"], L["mlp"]
        for b in ("1", "2") if f is not None else ("1",):
            out.update({p + "norm" + b: (), p + "rg" + b: (W, W), p + "rg" + b + ".b": (W,)})
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        if L["type"] == "attention":
            G, k = m["kv_heads"], m["conv"]
            for n, rows in (("q", 2 * H * d), ("k", 2 * G * d), ("v", G * dv)):
                out.update({f"{p}mix.{n}": (rows, W), f"{p}mix.{n}.conv": (rows, k)})
            out.update({p + "mix.q.norm": (d,), p + "mix.k.norm": (d,)})
            out.update({p + "mix." + n: (d,) for n in ("lq1", "lk1", "lq2", "lk2")})
        else:
            out.update({p + "mix.q": (H * d, W), p + "mix.f": (H * d, W), p + "mix.f.b": (H * d,), p + "mix.lower": (H * d,),
                        p + "mix.v": (H * dv, W), p + "mix.norm": (dv,)})
        out[p + "mix.o"] = (W, H * dv)
        if f is None:
            continue
        out[p + "mlp.router"] = (f["router"]["experts"], W)
        for e in range(f["router"]["experts"]):
            q = f"{p}mlp.e{e}."
            out.update({q + "gate": (f["expert"]["ff"], W), q + "up": (f["expert"]["ff"], W), q + "down": (W, f["expert"]["ff"])})
        if f.get("shared"):
            q, ff = p + "mlp.shared.", f["shared"]["ff"]
            out.update({q + "gate": (ff, W), q + "up": (ff, W), q + "down": (W, ff), q + "sg": (1, W)})
    return out


def random_weights(cfg: dict, seed: int, dtype=torch.bfloat16) -> Dict[str, torch.Tensor]:
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.split(".", 1)[1] if name.startswith("l") and name[1].isdigit() else name
        if leaf in ("norm1", "norm2", "final.norm"):
            t = 0.8 + 0.3 * torch.rand(shape, generator=g)
        elif leaf in ("mix.q.norm", "mix.k.norm", "mix.norm"):
            t = 1.0 + 0.2 * torch.randn(shape, generator=g)
        elif leaf.endswith(".conv"):
            t = torch.randn(shape, generator=g) / shape[1] ** 0.5
        elif leaf in ("mix.lq1", "mix.lk1", "mix.lq2", "mix.lk2"):
            t = torch.randn(shape, generator=g) * (0.4 / shape[0] ** 0.25)
        elif leaf == "mix.lower":
            t = 0.95 * torch.rand(shape, generator=g) ** 2
        elif leaf == "mix.f.b":
            t = 6.0 * torch.rand(shape, generator=g) - 1.0                  # (a channel forgets within a token to hundreds)
        elif leaf.endswith(".b"):
            t = 0.5 * torch.randn(shape, generator=g)
        elif leaf == "mlp.router":
            t = 2.0 * torch.randn(shape, generator=g) / shape[-1] ** 0.5
        elif name == "embed":
            t = torch.randn(shape, generator=g)
        else:
            t = torch.randn(shape, generator=g) / shape[-1] ** 0.5
        out[name] = t.to(dtype)
    return out


def write_model(folder: str, cfg: dict, seed: int) -> Dict[str, torch.Tensor]:
    from inferrs_amd.weights import write_safetensors
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    weights = random_weights(cfg, seed)
    write_safetensors(os.path.join(folder, "model.safetensors"), weights)
    return weights


def random_tokens(n: int, vocab: int, seed: int):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()
