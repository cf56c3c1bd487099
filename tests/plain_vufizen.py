"""A plain, slow implementation of the Vufizen decoder: whole sequences, no cache, no paging, no batching, one function
per mechanism, plain torch arithmetic on the CPU in one precision (float64 by default).  It shares no code with
`inferrs_amd`: a model is a config dictionary (the keys of config.json) and a dictionary of tensors by their names in
the file.

The design in short.  Both sub-layers read the stream as it stands; what one gives is multiplied by a sigmoid gate a
feature (a projection of that same stream, with a bias), RMS-normed with ONE weight for all features, and added:
x <- x + norm(sigmoid(W x + b) * sub(x)).  Two mixers.  "attention": differential attention, every head two maps with
queries and keys of their own over shared values, a1 - lambda a2 brought to unit root mean square a head and scaled by
1 - diff; q, k and v pass a short causal convolution a channel, q and k then an RMS norm a map and a turn by position
(neighbours paired).  "hgrn2": a matrix a head whose rows fade by a gate a channel and take in (gate's complement) v^T;
the read-out with silu(W_q x) is RMS-normed a head.  The feed-forward: routed gated-SiLU experts (softmax over the
chosen logits) beside a shared expert behind a sigmoid gate a token.  A layer may run another layer's tensors again.
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


def turn(x: torch.Tensor, positions: torch.Tensor, rot: Optional[dict]) -> torch.Tensor:
    """x [tokens, ..., dim]: of the first rot.dims features 2i turns with 2i + 1 by position * base^(-2i/dims)."""
    dims = int(rot["dims"]) if rot else 0
    if dims == 0:
        return x
    f = torch.tensor([float(rot["base"]) ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=x.dtype)
    a = positions.to(x.dtype)[:, None] * f[None, :]
    shape = (x.shape[0],) + (1,) * (x.dim() - 2) + (dims // 2,)
    c, s = torch.cos(a).view(shape), torch.sin(a).view(shape)
    out = x.clone()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * c - v * s
    out[..., 1:dims:2] = v * c + u * s
    return out


def short_convolution(u: torch.Tensor, taps: torch.Tensor) -> torch.Tensor:
    """u [tokens, channels], taps [channels, k]: y_t = sum_j taps[:, j] u_(t - k + 1 + j), zeros before the start."""
    n, k = u.shape[0], taps.shape[1]
    out = torch.zeros_like(u)
    for j in range(k):
        back = k - 1 - j
        if back < n:
            out[back:] += taps[:, j] * u[:n - back]
    return out


def softmax_rows(scores: torch.Tensor, seen: torch.Tensor) -> torch.Tensor:
    s = scores.masked_fill(~seen, float("-inf"))
    e = torch.exp(s - s.max(dim=-1, keepdim=True).values)
    return e / e.sum(dim=-1, keepdim=True)


# ---- the mixers -------------------------------------------------------------------------------

def map_weight(w: T, p: str, diff: float) -> torch.Tensor:
    """lambda: how much of the second map is taken off the first."""
    return torch.exp((w[p + "lq1"] * w[p + "lk1"]).sum()) - torch.exp((w[p + "lq2"] * w[p + "lk2"]).sum()) + diff


def differ(a1: torch.Tensor, a2: torch.Tensor, lam, diff: float, eps: float) -> torch.Tensor:
    return rms_norm(a1 - lam * a2, None, eps) * (1.0 - diff)


def differential_attention(h: torch.Tensor, w: T, p: str, m: dict, eps: float) -> torch.Tensor:
    n = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    diff = float(m["diff"])
    pos = torch.arange(n)
    q, k, v = (short_convolution(h @ w[p + x].T, w[p + x + ".conv"]) for x in ("q", "k", "v"))
    q = turn(rms_norm(q.view(n, H, 2, d), w[p + "q.norm"], eps), pos, m.get("rot"))
    k = turn(rms_norm(k.view(n, G, 2, d), w[p + "k.norm"], eps), pos, m.get("rot"))
    v = v.view(n, G, dv)
    seen = pos[:, None] >= pos[None, :]
    lam = map_weight(w, p, diff)
    out = torch.zeros(n, H, dv, dtype=h.dtype)
    for head in range(H):
        g = head // (H // G)
        a = [softmax_rows((q[:, head, j] @ k[:, g, j].T) * float(m["scale"]), seen) @ v[:, g] for j in range(2)]
        out[:, head] = differ(a[0], a[1], lam, diff, eps)
    return out.reshape(n, H * dv) @ w[p + "o"].T


def fading_outer_products(q: torch.Tensor, f: torch.Tensor, v: torch.Tensor, state: Optional[torch.Tensor] = None):
    """q, f [tokens, H, dim], v [tokens, H, vdim]: S <- diag(f) S + (1 - f) v^T from `state` [H, dim, vdim] (zero), o = S^T q.
    Returns (o [tokens, H, vdim], the last state)."""
    n, H, d = q.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=q.dtype) if state is None else state.clone()
    out = torch.zeros(n, H, v.shape[-1], dtype=q.dtype)
    for t in range(n):
        S = f[t][:, :, None] * S + (1.0 - f[t])[:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out, S


def hgrn2(h: torch.Tensor, w: T, p: str, m: dict, eps: float) -> torch.Tensor:
    n = h.shape[0]
    H, d, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q = silu(h @ w[p + "q"].T).view(n, H, d)
    lower = w[p + "lower"]
    f = (lower + (1.0 - lower) * torch.sigmoid(h @ w[p + "f"].T + w[p + "f.b"])).view(n, H, d)
    v = (h @ w[p + "v"].T).view(n, H, dv)
    o, _ = fading_outer_products(q, f, v)
    return rms_norm(o, w[p + "norm"], eps).reshape(n, H * dv) @ w[p + "o"].T


# ---- the feed-forward ---------------------------------------------------------------------------

def expert(h: torch.Tensor, w: T, p: str) -> torch.Tensor:
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(h: torch.Tensor, w: T, p: str, top: int):
    """(chosen experts [n, top], their weights [n, top]): the largest `top` logits, a softmax over those alone."""
    z = h @ w[p + "router"].T
    best = torch.topk(z, top, dim=-1)
    e = torch.exp(best.values - best.values.max(dim=-1, keepdim=True).values)
    return best.indices, e / e.sum(dim=-1, keepdim=True)


def routed_ff(h: torch.Tensor, w: T, p: str, f: dict) -> torch.Tensor:
    top = int(f["router"]["top"])
    chosen, weight = route(h, w, p, top)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for j in range(top):
            out[t] += weight[t, j] * expert(h[t:t + 1], w, f"{p}e{int(chosen[t, j])}.")[0]
    if f.get("shared"):
        out = out + expert(h, w, p + "shared.") * torch.sigmoid(h @ w[p + "shared.sg"].T)
    return out


# ---- the model ------------------------------------------------------------------------------------

def gated_branch(x: torch.Tensor, y: torch.Tensor, w: T, gate: str, norm: str, eps: float) -> torch.Tensor:
    """x + norm(y * sigmoid(W x + b)), the norm with one weight for all features."""
    return x + rms_norm(y * torch.sigmoid(x @ w[gate].T + w[gate + ".b"]), w[norm], eps)


def owner_of(layers: Sequence[dict], i: int) -> int:
    """The layer whose tensors layer i uses."""
    while layers[i].get("weights_of") is not None:
        i = int(layers[i]["weights_of"])
    return i


def forward(cfg: dict, w: T, tokens: Sequence[int], dtype=torch.float64, layers_out: Optional[List[torch.Tensor]] = None) -> torch.Tensor:
    """Logits [tokens, vocab] of one sequence from position 0.  `layers_out` receives the stream after every layer."""
    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in w.items()}
    eps = float(cfg["norm"]["eps"])
    x = w["embed"][torch.tensor(list(tokens), dtype=torch.long)]
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{owner_of(cfg['layers'], i)}.", layer["mixer"]
        mixer = {"attention": differential_attention, "hgrn2": hgrn2}[layer["type"]]
        x = gated_branch(x, mixer(x, w, p + "mix.", m, eps), w, p + "rg1", p + "norm1", eps)
        if layer.get("mlp") is not None:
            x = gated_branch(x, routed_ff(x, w, p + "mlp.", layer["mlp"]), w, p + "rg2", p + "norm2", eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T
