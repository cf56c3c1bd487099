"""Attention whose heads have two maps over shared values, the second taken off the first (differential attention; Ye et
al., "Differential Transformer"), behind a short convolution of queries, keys and values:

    q, k, v = conv(W_q h), conv(W_k h), conv(W_v h)                       (a channel each, zeros before a sequence's start)
    q, k <- turn(rmsnorm a map of a head)
    a1, a2 = softmax attention of either map over the same values;   lambda = exp(lq1 . lk1) - exp(lq2 . lk2) + diff
    out = W_o [ (a1 - lambda a2) / rms * (1 - diff) of every head ]

A key head's two maps lie side by side in the cache (a key of 2 * head_dim), and a map's query is as wide and zero
outside its own half: its product with the key head's row is the map's score, so the paged attention kernels run as
they are, with twice the query heads, and read every key and value once for both maps.  A request keeps the
convolution's last inputs, in 32-bit, beside its pages.
"""
from __future__ import annotations

import math
from typing import Dict

import torch

from .. import ops
from ..config.spec import AttentionSpec, DifferentialAttentionSpec, SpecError
from ..weights.loader import TensorSpec
from .attention import Attention
from .base import FixedState, Mixer, PagedAndState, PagedKV, part_class, register_mixer
from .linear import Linear, to_compute

MAPS = 2


@register_mixer("differential_attention")
class DifferentialAttention(Mixer):
    graph_safe = True
    lays_beside = True            # another matrix over the same input joins the projections' product (`lay_beside`)

    @classmethod
    def _channels(cls, spec: DifferentialAttentionSpec):
        return (spec.n_heads * MAPS * spec.head_dim, spec.n_kv_heads * MAPS * spec.head_dim, spec.n_kv_heads * spec.v_dim)

    @classmethod
    def tensors(cls, spec: DifferentialAttentionSpec) -> Dict[str, TensorSpec]:
        out: Dict[str, TensorSpec] = {}
        for name, rows in zip(("q", "k", "v"), cls._channels(spec)):
            out[name] = TensorSpec((rows, spec.hidden))
            out[name + ".conv"] = TensorSpec((rows, spec.conv))
        out["q.norm"] = out["k.norm"] = TensorSpec((spec.head_dim,), "norm")
        for name in ("lq1", "lk1", "lq2", "lk2"):
            out[name] = TensorSpec((spec.head_dim,))
        out["o"] = TensorSpec((spec.hidden, spec.n_heads * spec.v_dim))
        return out

    @classmethod
    def cache_need(cls, spec: DifferentialAttentionSpec):
        width = MAPS * spec.head_dim
        paged = PagedKV(spec.n_kv_heads, width, None, v_head_dim=spec.v_dim if spec.v_dim != width else None)
        if spec.conv <= 1:
            return paged
        return PagedAndState(paged, FixedState((cls._tail(spec),), torch.float32))       # the last inputs [conv - 1][channels]

    @classmethod
    def _tail(cls, spec: DifferentialAttentionSpec) -> int:
        floats = (spec.conv - 1) * sum(cls._channels(spec))
        return -(-floats // 4) * 4                   # (rows of whole 16-byte pieces)

    def __init__(self, spec: DifferentialAttentionSpec, tensors: Dict[str, torch.Tensor], dtype, device):
        if spec.n_heads % spec.n_kv_heads:
            raise SpecError(f"differential_attention: {spec.n_heads} heads are not a multiple of {spec.n_kv_heads} kv heads")
        if not (1 <= spec.head_dim <= 512 // MAPS) or not (1 <= spec.v_dim <= 512):
            raise SpecError(f"differential_attention: maps of {spec.head_dim} (up to {512 // MAPS}) and values of {spec.v_dim} (up to 512) "
                            "are the range of the attention kernels")
        rot = spec.position.rot_dim if spec.position.kind != "none" else 0
        if rot % 2 or rot > spec.head_dim:
            raise SpecError(f"differential_attention: the turned part of a map ({rot}) must be even and within {spec.head_dim}")
        if spec.conv < 1:
            raise SpecError(f"differential_attention: a convolution of {spec.conv} taps")
        self.spec = spec
        self.proj = Linear([tensors["q"], tensors["k"], tensors["v"]], dtype, device)
        self.o = Linear([tensors["o"]], dtype, device)
        # [taps, channels]: the kernel reads tap by tap
        self.taps = torch.cat([to_compute(tensors[n + ".conv"], dtype, device) for n in ("q", "k", "v")], dim=0).t().contiguous()
        self.q_norm_w, self.k_norm_w = (tensors[n].to(device=device, dtype=torch.float32).contiguous() for n in ("q.norm", "k.norm"))
        dot = lambda a, b: float((tensors[a].float() * tensors[b].float()).sum())
        self.lam = math.exp(dot("lq1", "lk1")) - math.exp(dot("lq2", "lk2")) + float(spec.diff)
        self.position = part_class("position", spec.position)(spec.position, {}, dtype, device)
        if getattr(self.position, "magnitude", 1.0) != 1.0:
            raise SpecError("differential_attention: a rotation law that scales cos and sin is not taken by this mixer's kernels")
        self.beside_off = None
        # (the attention kernels' launches are the attention part's: as many query heads as there are maps, keys of all maps)
        self.attend_spec = AttentionSpec(hidden=spec.hidden, n_heads=MAPS * spec.n_heads, n_kv_heads=spec.n_kv_heads,
                                         head_dim=MAPS * spec.head_dim, position=spec.position, scale=spec.scale, v_head_dim=spec.v_dim)

    def lay_beside(self, weight: torch.Tensor) -> None:
        """Stack `weight` [features, hidden] behind the projections: its product is left in `ctx.beside`."""
        w = self.proj.weight
        self.beside_off = w.shape[0]
        self.proj = Linear([w, weight], w.dtype, w.device)

    def forward(self, ctx, h, cache):
        s = self.spec
        group = ctx.groups[cache.group]
        if hasattr(h, "materialize"):
            h = h.materialize()
        proj = self.proj(h)                                      # [n, q | k | v | what is laid beside]
        if self.beside_off is not None:
            ctx.beside = (proj, self.beside_off)
        table = ctx.position_table(self.position)
        cos, sin = table if table is not None else (None, None)
        q = ops.conv_qkv(proj, self.taps, cache.state, 0, heads=s.n_heads, kv_heads=s.n_kv_heads, maps=MAPS, dim=s.head_dim,
                         vdim=s.v_dim, q_norm_w=self.q_norm_w, k_norm_w=self.k_norm_w, eps=s.norm_eps, cos=cos, sin=sin,
                         rot=self.position.rot_dim, interleaved=self.position.interleaved, k_cache=cache.k, v_cache=cache.v,
                         slots=group.slots, page_size=group.page_size, token_seq=ctx.token_seq, cu_tokens=ctx.cu_tokens,
                         state_slots=ctx.state_slots, max_q_len=ctx.max_q_len)
        a = Attention.attend(self.attend_spec, ctx, q, cache, group)
        joined = ops.differ_norm(a, self.lam, s.norm_eps, 1.0 - s.diff)
        if getattr(ctx, "partial_sums", False):
            split = ops.linear_partials(joined, self.o.weight)
            if split is not None:
                return split
        return self.o(joined)
