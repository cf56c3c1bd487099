"""Tiny Lumedra configurations that differ in every size and option, and random weights for them.

The tensor list is written out here from the design (not asked of the package), so a part that expects another name or
shape fails to load.  Weights are drawn so that the mechanisms matter: matrices N(0, 1/in), norm weights away from 1, value
mixtures of a third and more, router logits that spread.  `sharpened` multiplies every attention's `scale` so that a query
singles out a few keys, and a key that is lost, hidden or read from a wrong page changes the logits by far more than rounding."""
from __future__ import annotations

import copy
import json
import os
from typing import Dict

import torch


def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, base=10000.0):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank,
                                                  "kv_rank": kv_rank, "scale": scale, "rot": {"base": base, "dims": rot_dim}}}


def lightning(heads, dim, vdim, decay):
    assert len(decay) == heads
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}}


def attn(heads, kv_heads, dim, vdim, scale, size=None, keep_first=0, softcap=None, v_mix=False):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if size is not None:
        m["mask"] = {"size": size, "keep_first": keep_first}
    if softcap is not None:
        m["softcap"] = softcap
    if v_mix:
        m["v_mix"] = True
    return {"type": "attention", "mixer": m}


def dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(experts, top, ff, scale=1.0, groups=None, shared=None):
    f = {"kind": "moe", "router": {"experts": experts, "top": top, "scale": scale}, "expert": {"ff": ff}}
    if groups is not None:
        f["router"]["groups"] = {"count": groups[0], "keep": groups[1]}
    if shared is not None:
        f["shared"] = {"ff": shared}
    return f


def layer(mixer, mlp):
    return {**mixer, "mlp": mlp}


def model(vocab, width, layers, eps=1e-6):
    return {"architecture": "Lumedra", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


# A: all three mixers, three layers that mix values (heads of their own each), one attention that does not between them, windows of
# two sizes with kept first tokens inside a page and over pages, a dense layer, a layer without feed-forward.
CFG_A = model(199, 48, [layer(attn(4, 2, 10, 12, 0.4, size=20, keep_first=5, softcap=8.0, v_mix=True), moe(6, 2, 24, 2.5, (3, 2), 16)),
                        layer(latent(3, 12, 6, 14, 20, 26, 0.3, 500.0), dense(40, 0.8)),
                        layer(lightning(3, 12, 10, (0.4, 0.9, 0.998)), moe(8, 3, 16, 1.5, (4, 2))),
                        layer(attn(3, 3, 14, 8, 0.35, size=11, keep_first=37, softcap=3.0), None),
                        layer(attn(2, 2, 16, 12, 0.3, size=70, keep_first=1, softcap=20.0, v_mix=True), dense(24, 2.0)),
                        layer(attn(6, 2, 8, 12, 0.4, size=20, keep_first=5, v_mix=True), moe(5, 1, 16, 0.7, None, 8))], eps=1e-5)
# B: every count 1 and every size equal where the design lets them differ; one expert, one group, nothing kept, no cap.
CFG_B = model(97, 64, [layer(latent(1, 64, 64, 64, 64, 64, 0.125), moe(1, 1, 64, 1.0, (1, 1), 64)),
                       layer(attn(1, 1, 64, 64, 0.125, size=1, keep_first=0, v_mix=True), moe(2, 2, 64, 1.0, (2, 2))),
                       layer(lightning(1, 64, 64, (1.0,)), dense(64, 1.0))])
# C: sizes that fit no vector width: a width of 50, heads of 11 and 13, a latent row of 21 + 2, states of 10 x 7 and 21 x 33,
# feed-forwards of 30 and 22; a window shorter than what is kept.
CFG_C = model(101, 50, [layer(lightning(5, 10, 7, (0.0, 0.2, 0.7, 0.95, 1.0)), moe(9, 4, 30, 3.0, (3, 3), 22)),
                        layer(latent(3, 11, 2, 13, 17, 21, 0.5, 777.0), moe(6, 3, 22, 1.0, (2, 1))),
                        layer(attn(3, 3, 11, 13, 0.5, size=6, keep_first=19, softcap=5.0, v_mix=True), dense(30, 0.5)),
                        layer(lightning(2, 21, 33, (0.5, 0.99)), None),
                        layer(attn(6, 3, 13, 13, 0.5, size=33, keep_first=33, softcap=5.0, v_mix=True), moe(3, 3, 30))], eps=1e-5)
# D: the matrix cores' sizes with long sequences: a latent row of 112 + 16 and heads of 128 and 64 with windows across several
# stages of keys, a state of 128 x 128 and one of 32 x 160, sixty-four experts in eight groups.
CFG_D = model(150, 128, [layer(latent(4, 32, 16, 48, 64, 112, 0.2, 30000.0), moe(64, 6, 32, 2.0, (8, 3), 16)),
                         layer(attn(4, 2, 128, 128, 0.1, size=100, keep_first=70, softcap=6.0, v_mix=True), moe(4, 1, 64, 1.0, (2, 1))),
                         layer(lightning(2, 128, 128, (0.9, 0.999)), dense(96, 1.5)),
                         layer(attn(8, 4, 64, 64, 0.15, size=200, keep_first=130, v_mix=True), None),
                         layer(lightning(3, 32, 160, (0.05, 0.97, 1.0)), moe(6, 2, 32, 1.0, (3, 2), 32)),
                         layer(attn(4, 4, 32, 32, 0.2, size=130, keep_first=16, softcap=10.0), dense(64, 1.0))])
# E: keys too wide for the chunks (the recurrence walks a prompt) and a single column, attention over every earlier key with capped
# scores, and without caps or windows at all.
CFG_E = model(83, 40, [layer(lightning(2, 150, 20, (0.8, 0.99)), moe(3, 1, 16)),
                       layer(attn(2, 1, 24, 48, 0.3, softcap=4.0, v_mix=True), moe(4, 2, 24, 1.2, (2, 2), 8)),
                       layer(lightning(4, 1, 24, (0.1, 0.6, 0.9, 0.9)), dense(8, 3.0)),
                       layer(attn(2, 2, 48, 24, 0.3, v_mix=True), moe(2, 2, 8, 2.0))])
# F: no layer that caches keys at all.
CFG_F = model(61, 32, [layer(lightning(2, 16, 16, (0.9, 0.5)), dense(48, 0.7)), layer(lightning(1, 40, 24, (0.98,)), moe(4, 2, 16, 1.0, (2, 1)))])
CONFIGS = {"A": CFG_A, "B": CFG_B, "C": CFG_C, "D": CFG_D, "E": CFG_E, "F": CFG_F}


def sharpened(cfg: dict, factor: float) -> dict:
    """The same model with every attention's `scale` multiplied (and its cap): its queries single out few of the keys they see."""
    out = copy.deepcopy(cfg)
    for L in out["layers"]:
        if L["type"] != "lightning":
            L["mixer"]["scale"] = L["mixer"]["scale"] * factor
            if L["mixer"].get("softcap") is not None:
                L["mixer"]["softcap"] = L["mixer"]["softcap"] * factor
    return out


def tensor_shapes(cfg: dict) -> Dict[str, tuple]:
    """Every tensor of a model, from the design."""
    W, V = cfg["width"], cfg["vocab"]
    out = {"embed": (V, W), "final.norm": (W,)}
    mixed_before = False
    for i, L in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", L["mixer"], L["mlp"]
        out[p + "norm1"] = (W,)
        if f is not None:
            out[p + "norm2"] = (W,)
        q = p + "mix."
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        out[q + "o"] = (W, H * dv)
        if L["type"] == "latent_attention":
            r, rank = m["rot_dim"], m["kv_rank"]
            out.update({q + "dq": (m["q_rank"], W), q + "dq.norm": (m["q_rank"],), q + "uq": (H * (d + r), m["q_rank"]),
                        q + "dkv": (rank + r, W), q + "dkv.norm": (rank,), q + "uk": (H * d, rank), q + "uv": (H * dv, rank),
                        q + "g": (H * dv, W)})
        elif L["type"] == "lightning":
            out.update({q + "q": (H * d, W), q + "k": (H * d, W), q + "v": (H * dv, W), q + "g": (H * dv, W), q + "norm": (H * dv,)})
        else:
            G = m["kv_heads"]
            out.update({q + "q": (H * d, W), q + "k": (G * d, W), q + "v": (G * dv, W)})
            if m.get("v_mix"):
                if mixed_before:                  # (a file holds the first such layer's number too; nothing reads it)
                    out[q + "vmix"] = ()
                mixed_before = True
        if f is None:
            continue
        if f["kind"] == "dense":
            out.update({p + "mlp.gate": (f["ff"], W), p + "mlp.up": (f["ff"], W), p + "mlp.down": (W, f["ff"])})
            continue
        out[p + "mlp.router"] = (f["router"]["experts"], W)
        for e in range(f["router"]["experts"]):
            q = f"{p}mlp.e{e}."
            out.update({q + "gate": (f["expert"]["ff"], W), q + "up": (f["expert"]["ff"], W), q + "down": (W, f["expert"]["ff"])})
        if f.get("shared"):
            q, ff = p + "mlp.shared.", f["shared"]["ff"]
            out.update({q + "gate": (ff, W), q + "up": (ff, W), q + "down": (W, ff)})
    return out


def random_weights(cfg: dict, seed: int, dtype=torch.bfloat16) -> Dict[str, torch.Tensor]:
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.split(".", 1)[1] if name.startswith("l") and name[1].isdigit() else name
        if leaf in ("norm1", "norm2", "final.norm", "mix.norm", "mix.dq.norm", "mix.dkv.norm"):
            t = 1.0 + 0.25 * torch.randn(shape, generator=g)
        elif leaf == "mix.vmix":
            t = 0.35 + 0.4 * torch.rand(shape, generator=g)
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
    stored = dict(weights)
    for i, L in enumerate(cfg["layers"]):         # the first mixing layer's own number: in the file, and of no consequence
        if L["type"] == "attention" and L["mixer"].get("v_mix"):
            stored[f"l{i}.mix.vmix"] = torch.tensor(7.0, dtype=torch.bfloat16)
            break
    stored.update({k: v for k, v in weights.items() if k.endswith(".vmix")})
    write_safetensors(os.path.join(folder, "model.safetensors"), stored)
    return weights


def random_tokens(n: int, vocab: int, seed: int):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()
