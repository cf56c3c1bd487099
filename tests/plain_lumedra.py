"""A plain, slow implementation of the Lumedra decoder: whole sequences, no cache, no paging, no batching, one function
per mechanism, plain torch arithmetic on the CPU in one precision (float64 by default).  It shares no code with
`inferrs_amd`: a model is a config dictionary (the keys of config.json) and a dictionary of tensors by their names in
the file.

The design in short.  A layer adds two sub-layers to the stream at once, each behind an RMS norm of its own of the same
rows: x <- x + mixer(norm1(x)) + ff(norm2(x)).  Three mixers.  "latent_attention": queries, keys and values out of
low-rank rows, one turned key part for all heads, every earlier key, a sigmoid gate a feature.  "lightning": a matrix a
head that fades by a constant and takes in silu(k) silu(v)^T, one RMS norm over all heads' outputs, a sigmoid gate.
"attention": grouped heads without a turn, capped scores, a window beside the first few tokens, values that are mixed
with those of the first layer that mixes.  Feed-forwards: a clamped dense one, or routed gated-SiLU experts chosen by
sigmoid scores inside the best groups, beside a shared one.  Logits through the embedding table.
"""
from __future__ import annotations

from typing import Dict, List, Optional, Sequence

import torch

T = Dict[str, torch.Tensor]


# ---- small pieces ---------------------------------------------------------------------------

def rms_norm(x: torch.Tensor, w, eps: float) -> torch.Tensor:
    y = x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)
    return y if w is None else y * w


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def turn(x: torch.Tensor, positions: torch.Tensor, base: float) -> torch.Tensor:
    """x [tokens, ..., dims]: feature 2i turns with 2i + 1 by position * base^(-2i/dims)."""
    dims = x.shape[-1]
    if dims == 0:
        return x
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=x.dtype)
    a = positions.to(x.dtype)[:, None] * f[None, :]
    shape = (x.shape[0],) + (1,) * (x.dim() - 2) + (dims // 2,)
    c, s = torch.cos(a).view(shape), torch.sin(a).view(shape)
    u, v = x[..., 0::2], x[..., 1::2]
    return torch.stack([u * c - v * s, v * c + u * s], dim=-1).reshape(x.shape)


def softmax_rows(scores: torch.Tensor, seen: torch.Tensor) -> torch.Tensor:
    s = scores.masked_fill(~seen, float("-inf"))
    e = torch.exp(s - s.max(dim=-1, keepdim=True).values)
    return e / e.sum(dim=-1, keepdim=True)


# ---- the mixers -------------------------------------------------------------------------------

def latent_attention(h: torch.Tensor, w: T, p: str, m: dict, eps: float) -> torch.Tensor:
    n = h.shape[0]
    H, d, r, dv, rank = (int(m[k]) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
    pos = torch.arange(n)
    base = float(m["rot"]["base"])
    q = (rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps) @ w[p + "uq"].T).view(n, H, d + r)
    down = h @ w[p + "dkv"].T
    c = rms_norm(down[:, :rank], w[p + "dkv.norm"], eps)
    k_rot = turn(down[:, rank:], pos, base)
    k = (c @ w[p + "uk"].T).view(n, H, d)
    v = (c @ w[p + "uv"].T).view(n, H, dv)
    q_rot = turn(q[:, :, d:], pos, base)
    seen = pos[:, None] >= pos[None, :]
    out = torch.zeros(n, H, dv, dtype=h.dtype)
    for head in range(H):
        s = (q[:, head, :d] @ k[:, head].T + q_rot[:, head] @ k_rot.T) * float(m["scale"])
        out[:, head] = softmax_rows(s, seen) @ v[:, head]
    return (out.reshape(n, H * dv) * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def fading_sums(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay: Sequence[float], state: Optional[torch.Tensor] = None):
    """q, k [tokens, H, dim], v [tokens, H, vdim]: S <- decay_h S + k v^T from `state` [H, dim, vdim] (zero), o = S^T q.
    Returns (o [tokens, H, vdim], the last state)."""
    n, H, d = q.shape
    a = torch.tensor(list(decay), dtype=q.dtype)[:, None, None]
    S = torch.zeros(H, d, v.shape[-1], dtype=q.dtype) if state is None else state.clone()
    out = torch.zeros(n, H, v.shape[-1], dtype=q.dtype)
    for t in range(n):
        S = a * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out, S


def lightning(h: torch.Tensor, w: T, p: str, m: dict, eps: float) -> torch.Tensor:
    n = h.shape[0]
    H, d, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q, k = (silu(h @ w[p + x].T).view(n, H, d) for x in ("q", "k"))
    v = silu(h @ w[p + "v"].T).view(n, H, dv)
    o, _ = fading_sums(q, k, v, m["decay"])
    return (rms_norm(o.reshape(n, H * dv), w[p + "norm"], eps) * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def seen_keys(n: int, mask: Optional[dict]) -> torch.Tensor:
    """[query, key]: the last mask.size positions, itself included, and the first mask.keep_first; no mask: every earlier one."""
    i = torch.arange(n)
    far = i[:, None] - i[None, :]
    seen = far >= 0
    if mask:
        seen = seen & ((far < int(mask["size"])) | (i[None, :] < int(mask.get("keep_first", 0))))
    return seen


def capped(scores: torch.Tensor, cap: Optional[float]) -> torch.Tensor:
    return scores if cap is None else cap * torch.tanh(scores / cap)


def mixed_values(v: torch.Tensor, first: torch.Tensor, lam) -> torch.Tensor:
    return (1.0 - lam) * v + lam * first


def grouped_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, cap: Optional[float], seen: torch.Tensor) -> torch.Tensor:
    """q [n, H, d], k [n, G, d], v [n, G, dv] -> [n, H, dv]."""
    n, H, G = q.shape[0], q.shape[1], k.shape[1]
    out = torch.zeros(n, H, v.shape[-1], dtype=q.dtype)
    for head in range(H):
        g = head // (H // G)
        out[:, head] = softmax_rows(capped((q[:, head] @ k[:, g].T) * scale, cap), seen) @ v[:, g]
    return out


def attention(h: torch.Tensor, w: T, p: str, m: dict, v_first: List[torch.Tensor]) -> torch.Tensor:
    """`v_first`: empty until the first layer that mixes values has left its own there."""
    n = h.shape[0]
    H, G, d = int(m["heads"]), int(m["kv_heads"]), int(m["dim"])
    dv = int(m["vdim"])
    q, k, v = h @ w[p + "q"].T, h @ w[p + "k"].T, h @ w[p + "v"].T
    if m.get("v_mix"):
        if v_first:
            v = mixed_values(v, v_first[0], w[p + "vmix"])
        else:
            v_first.append(v)
    cap = m.get("softcap")
    out = grouped_attention(q.view(n, H, d), k.view(n, G, d), v.view(n, G, dv), float(m["scale"]),
                            None if cap is None else float(cap), seen_keys(n, m.get("mask")))
    return out.reshape(n, H * dv) @ w[p + "o"].T


# ---- the feed-forwards --------------------------------------------------------------------------

def clamped_ff(h: torch.Tensor, w: T, p: str, limit: float) -> torch.Tensor:
    g = (h @ w[p + "gate"].T).clamp(max=limit)
    u = (h @ w[p + "up"].T).clamp(-limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].T


def silu_ff(h: torch.Tensor, w: T, p: str) -> torch.Tensor:
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def best_groups(s: torch.Tensor, count: int, keep: int) -> torch.Tensor:
    """[n, experts] scores -> which experts lie in the `keep` of `count` neighbouring groups with the largest sums of two."""
    n, E = s.shape
    size = E // count
    in_groups = s.view(n, count, size)
    worth = torch.sort(in_groups, dim=-1, descending=True).values[:, :, :2].sum(-1)
    best = torch.topk(worth, keep, dim=-1).indices
    allowed = torch.zeros(n, count, dtype=torch.bool).scatter_(1, best, True)
    return allowed[:, :, None].expand(n, count, size).reshape(n, E)


def route(h: torch.Tensor, w: T, p: str, router: dict):
    """(chosen experts [n, top], their weights [n, top])."""
    s = torch.sigmoid(h @ w[p + "router"].T)
    key, groups = s, router.get("groups")
    if groups:
        key = s.masked_fill(~best_groups(s, int(groups["count"]), int(groups["keep"])), float("-inf"))
    chosen = torch.topk(key, int(router["top"]), dim=-1).indices
    won = torch.gather(s, 1, chosen)
    return chosen, won / (won.sum(-1, keepdim=True) + 1e-20) * float(router.get("scale", 1.0))


def routed_ff(h: torch.Tensor, w: T, p: str, f: dict) -> torch.Tensor:
    chosen, weight = route(h, w, p, f["router"])
    out = torch.zeros_like(h)
    for e in range(int(f["router"]["experts"])):
        t, j = torch.nonzero(chosen == e, as_tuple=True)
        if t.numel():
            out[t] += weight[t, j][:, None] * silu_ff(h[t], w, f"{p}e{e}.")
    if f.get("shared"):
        out = out + silu_ff(h, w, p + "shared.")
    return out


def feed_forward(h: torch.Tensor, w: T, p: str, f: dict) -> torch.Tensor:
    return clamped_ff(h, w, p, float(f["limit"])) if f["kind"] == "dense" else routed_ff(h, w, p, f)


# ---- the model ------------------------------------------------------------------------------------

def forward(cfg: dict, w: T, tokens: Sequence[int], dtype=torch.float64, layers_out: Optional[List[torch.Tensor]] = None) -> torch.Tensor:
    """Logits [tokens, vocab] of one sequence from position 0.  `layers_out` receives the stream after every layer."""
    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in w.items()}
    eps = float(cfg["norm"]["eps"])
    x = w["embed"][torch.tensor(list(tokens), dtype=torch.long)]
    v_first: List[torch.Tensor] = []
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h = rms_norm(x, w[p + "norm1"], eps)
        if layer["type"] == "attention":
            y = attention(h, w, p + "mix.", m, v_first)
        else:
            y = {"latent_attention": latent_attention, "lightning": lightning}[layer["type"]](h, w, p + "mix.", m, eps)
        if layer.get("mlp") is not None:
            y = y + feed_forward(rms_norm(x, w[p + "norm2"], eps), w, p + "mlp.", layer["mlp"])
        x = x + y
        if layers_out is not None:
            layers_out.append(x.clone())
    return rms_norm(x, w["final.norm"], eps) @ w["embed"].T
