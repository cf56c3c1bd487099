"""A mixer that carries a matrix a head whose ROWS fade, each by a gate of its own a token, and take in what the gate leaves
open (HGRN2; Qin et al., "HGRN2: Gated Linear RNNs with State Expansion"):

    f = lower + (1 - lower) * sigmoid(W_f h + b)                  (a gate a channel, `lower` its learned floor)
    S_t = diag(f_t) S_(t-1) + (1 - f_t) v_t^T,   o_t = S_t^T silu(W_q h)_t
    out = W_o [ o / rms * w of every head ]                       (one weight of v_dim entries for all heads)

A request keeps its matrices in its row of a fixed-size 32-bit state array; gates, recurrence and norm are 32-bit whatever
the products' precision (`ops.fading_scan`)."""
from __future__ import annotations

from typing import Dict

import torch

from .. import ops
from ..config.spec import FadingStateSpec, SpecError
from ..weights.loader import TensorSpec
from .base import FixedState, Mixer, register_mixer
from .linear import Linear


@register_mixer("hgrn2")
class FadingState(Mixer):
    graph_safe = True
    lays_beside = True            # another matrix over the same input joins the projections' product (`lay_beside`)

    @classmethod
    def tensors(cls, spec: FadingStateSpec) -> Dict[str, TensorSpec]:
        qk, vv = spec.n_heads * spec.head_dim, spec.n_heads * spec.v_dim
        return {"q": TensorSpec((qk, spec.hidden)), "f": TensorSpec((qk, spec.hidden)), "f.b": TensorSpec((qk,)),
                "lower": TensorSpec((qk,)), "v": TensorSpec((vv, spec.hidden)), "norm": TensorSpec((spec.v_dim,), "norm"),
                "o": TensorSpec((spec.hidden, vv))}

    @classmethod
    def cache_need(cls, spec: FadingStateSpec):
        floats = spec.n_heads * spec.v_dim * spec.head_dim             # the matrices [heads][v_dim][dim]
        return FixedState((-(-floats // 4) * 4,), torch.float32)       # (rows of whole 16-byte pieces)

    def __init__(self, spec: FadingStateSpec, tensors: Dict[str, torch.Tensor], dtype, device):
        if not (1 <= spec.head_dim <= ops.gated.FADING_MAX_DIM):
            raise SpecError(f"hgrn2: a key size of {spec.head_dim} is outside 1..{ops.gated.FADING_MAX_DIM}, the range of the recurrence kernel")
        self.spec = spec
        self.proj = Linear([tensors["q"], tensors["f"], tensors["v"]], dtype, device)
        self.o = Linear([tensors["o"]], dtype, device)
        self.f_bias, self.lower, self.norm = (tensors[n].to(device=device, dtype=torch.float32).contiguous() for n in ("f.b", "lower", "norm"))
        self.beside_off = None

    def lay_beside(self, weight: torch.Tensor) -> None:
        """Stack `weight` [features, hidden] behind the projections: its product is left in `ctx.beside`."""
        w = self.proj.weight
        self.beside_off = w.shape[0]
        self.proj = Linear([w, weight], w.dtype, w.device)

    def forward(self, ctx, h, cache):
        s = self.spec
        qk = s.n_heads * s.head_dim
        if hasattr(h, "materialize"):
            h = h.materialize()
        proj = self.proj(h)                                      # [n, q | f | v | what is laid beside]
        if self.beside_off is not None:
            ctx.beside = (proj, self.beside_off)
        y = ops.fading_scan(proj, q_off=0, f_off=qk, v_off=2 * qk, heads=s.n_heads, dim=s.head_dim, vdim=s.v_dim, f_bias=self.f_bias,
                            lower=self.lower, norm_weight=self.norm, eps=s.norm_eps, state=cache.state, s_off=0,
                            cu_tokens=ctx.cu_tokens, state_slots=ctx.state_slots, max_q_len=ctx.max_q_len)
        if getattr(ctx, "partial_sums", False):
            split = ops.linear_partials(y, self.o.weight)
            if split is not None:
                return split
        return self.o(y)
