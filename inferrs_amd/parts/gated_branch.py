"""A layer whose sub-layers read a 32-bit residual stream as it stands, each output gated and normed before it enters:

    x <- x + norm_a(mixer(x) * sigmoid(W_a x + b_a));   x <- x + norm_b(ffn(x) * sigmoid(W_b x + b_b))
                                                       (a layer may lack the feed-forward, an arrangement the gates)

The stream that this arrangement hands from block to block is the 32-bit array [tokens, width]; beside it goes the same
array once more in the products' precision (`ctx.post_rows`: what the next sub-layer's products read; in a 32-bit model the
stream itself).  One kernel closes a sub-layer (`ops.branch_step`): it adds the parts of the output up (a dense one, one
still split along its k, the weighted rows of routed experts, a shared expert's output times its gate a token), gates, norms
and adds the result, and writes both arrays.  A block leaves nothing to be added.

The mixer's gate reads what the mixer's own projection reads: a mixer with `lays_beside` takes the gate's matrix into its
product (`lay_beside`, once, when the block is built) and leaves (rows, offset) in `ctx.beside` when it runs.  The feed-forward's
gate and a router's matrix read the same rows too: steps of a few rows form gate and logits in one product with 32-bit
results (`ctx.router_logits`), longer ones apart (the gate in the products' precision, the logits in 32-bit by the
router's own kernel).
"""
from __future__ import annotations

from typing import Dict, Tuple

import torch

from .. import ops
from ..config.spec import GatedBranchSpec, LayerSpec, SpecError
from ..weights.loader import TensorSpec
from .base import BlockBase, part_class, register_block
from .block import sub_tensors
from .experts import RoutedRows
from .linear import Linear
from .norm import build_norm, norm_tensors


@register_block("gated_branch")
class GatedBranchBlock(BlockBase):
    graph_safe = True

    @classmethod
    def tensors(cls, spec: LayerSpec) -> Dict[str, TensorSpec]:
        branches = 1 if spec.ffn is None else 2
        gates, suffix = cls._gates(spec)
        if len(spec.norms) != branches or len(spec.norm_names) != branches or (gates is not None and len(gates) != branches):
            raise SpecError(f"the arrangement 'gated_branch' has {branches} norms and as many gates here, the layer names {len(spec.norms)}")
        out: Dict[str, TensorSpec] = {}
        for local, ts in part_class("mixer", spec.mixer).tensors(spec.mixer).items():
            out[spec.mixer_prefix + local] = ts
        if spec.ffn is not None:
            for local, ts in part_class("ffn", spec.ffn).tensors(spec.ffn).items():
                out[spec.ffn_prefix + local] = ts
        for name, nspec in zip(spec.norm_names, spec.norms):
            out.update(norm_tensors(name, nspec))
        width = spec.norms[0].size
        for name in gates or ():
            out[name] = TensorSpec((width, width))
            out[name + suffix] = TensorSpec((width,))
        return out

    @staticmethod
    def _gates(spec: LayerSpec):
        residual = spec.residual if spec.residual is not None else GatedBranchSpec()
        if not isinstance(residual, GatedBranchSpec):
            raise SpecError("gated_branch: the layer's `residual` is a GatedBranchSpec")
        return residual.gate_names, residual.bias_suffix

    def __init__(self, spec: LayerSpec, tensors: Dict[str, torch.Tensor], dtype, device):
        self.spec, self.dtype = spec, dtype
        self.mixer = part_class("mixer", spec.mixer)(spec.mixer, sub_tensors(tensors, spec.mixer_prefix), dtype, device)
        self.ffn = None
        if spec.ffn is not None:
            self.ffn = part_class("ffn", spec.ffn)(spec.ffn, sub_tensors(tensors, spec.ffn_prefix), dtype, device)
        self.norms = [build_norm(name, nspec, tensors, dtype, device) for name, nspec in zip(spec.norm_names, spec.norms)]
        for n in self.norms:
            if getattr(n, "add_one", False) or getattr(n, "kind", "") != "rmsnorm":
                raise SpecError("gated_branch: the norms must be plain RMS norms")
        self.first_norm = None                      # (no norm reads the stream ahead of this block's parts)
        names, suffix = self._gates(spec)
        names = names or ()
        self.gate_bias_mixer = self.gate_bias_ffn = self.gate_mixer = self.gate_ffn = None
        biases = [tensors[name + suffix].to(device=device, dtype=torch.float32).contiguous() for name in names]
        if names:
            self.gate_bias_mixer = biases[0]
            if getattr(self.mixer, "lays_beside", False):
                self.mixer.lay_beside(Linear([tensors[names[0]]], dtype, device).weight)
            else:
                self.gate_mixer = Linear([tensors[names[0]]], dtype, device)
        if len(names) > 1:
            self.gate_bias_ffn = biases[1]
            weights = [Linear([tensors[names[1]]], dtype, device).weight]
            if getattr(self.ffn, "takes_logits", False) and dtype == torch.bfloat16:
                # the router's rows behind the gate's: steps of a few rows form both in one product with 32-bit results
                # (padded with rows of zeros: the result's rows then start at multiples of 16 bytes)
                pad = -(weights[0].shape[0] + self.ffn.router.shape[0]) % 8
                weights += [self.ffn.router, torch.zeros((pad, weights[0].shape[1]), dtype=dtype, device=weights[0].device)]
            self.gate_ffn = torch.cat(weights, dim=0).contiguous()
            self.gate_rows = weights[0].shape[0]
            if len(weights) > 1:
                self.ffn.router = self.gate_ffn[self.gate_rows:self.gate_rows + self.ffn.router.shape[0]]

    def parts(self):
        return [self, self.mixer, self.ffn, *self.norms, getattr(self.mixer, "position", None),
                *getattr(self.mixer, "parts", lambda: [])(), getattr(self.ffn, "shared", None)]

    # ---- the model's two ends ---------------------------------------------------------------------
    def enter(self, ctx, rows: torch.Tensor) -> torch.Tensor:
        """The embedding's rows -> the 32-bit stream; the rows in the products' precision go beside it."""
        if rows.dtype == torch.float32:
            if self.dtype == torch.float32:
                ctx.post_rows = rows
            return rows                              # (an embedding that leaves 32-bit rows has put the others into ctx.post_rows)
        ctx.post_rows = rows
        return ops.widen(rows)

    def leave(self, ctx, x: torch.Tensor, pending, rows: torch.Tensor, norm) -> torch.Tensor:
        """The final norm of the wanted rows (the last block has left nothing to be added)."""
        if pending is not None:
            raise SpecError("gated_branch: the block before leaves something that this arrangement does not take")
        if norm is None or getattr(norm, "add_one", False) or getattr(norm, "kind", "") != "rmsnorm":
            raise SpecError("gated_branch: the model ends with a plain RMS norm")
        ctx.post_rows = None
        return ops.parallel_step(x, rows=rows, norm_weight=norm.weight, norm_eps=norm.eps, center=False, h_dtype=self.dtype)[1]

    # ---- a layer ------------------------------------------------------------------------------------
    def _close(self, x: torch.Tensor, out, norm, gate, bias):
        """x <- x + norm(out * sigmoid(gate + bias)); returns what the next products read."""
        if isinstance(out, RoutedRows):
            if out.sel is not None or out.weights is None:
                raise SpecError("gated_branch: experts that hand their input on, and weights on the experts' inputs, are not "
                                "taken by this arrangement")
            adds = dict(routed=out.rows, routed_weights=out.weights, y3=_dense(out.extra), y3_scale=out.extra_scale)
        else:
            adds = dict(y=_dense(out))
        if gate is not None:
            adds.update(gate=gate[0], gate_off=gate[1], gate_bias=bias)
        xr = ops.branch_step(x, weight=norm.weight, eps=norm.eps, x_dtype=None if self.dtype == torch.float32 else self.dtype, **adds)
        return x if xr is None else xr

    def _ffn_gate(self, ctx, h):
        """The feed-forward's gate; in steps of a few rows the router's logits with it (`ctx.router_logits`)."""
        ctx.router_logits = None
        if self.gate_ffn is None:
            return None
        if self.gate_ffn.shape[0] > self.gate_rows:
            if h.shape[0] <= min(ops.mix.ROUTE_LOGITS_ROWS, ops.SKINNY_MAX_ROWS) and ops.skinny_fits(h, self.gate_ffn):
                rows = ops.linear(h, self.gate_ffn, torch.float32)
                ctx.router_logits = (rows, self.gate_rows)
                return rows, 0
        return ops.linear(h, self.gate_ffn[:self.gate_rows]), 0

    def forward(self, ctx, x: torch.Tensor, pending, cache, next_norm=None) -> Tuple[torch.Tensor, object]:
        if x.dim() != 2 or x.dtype != torch.float32:
            raise SpecError(f"gated_branch: the block takes a 32-bit stream [tokens, width], got {tuple(x.shape)} {x.dtype}")
        if pending is not None:
            raise SpecError("gated_branch: the block before leaves something that this arrangement does not take")
        ctx.stream = ctx.stream_norm = None
        # steps of few rows: a part's last product may stay split along k (gemm_mid.hip), for `ops.branch_step` to add up
        ctx.partial_sums = self.dtype == torch.bfloat16 and ops.MID_MIN_ROWS <= x.shape[0] <= ops.MID_MAX_ROWS
        h = getattr(ctx, "post_rows", None)
        if h is None or h.shape != x.shape:
            h = x if self.dtype == torch.float32 else x.to(self.dtype)
        ctx.beside = None
        out = self.mixer.forward(ctx, h, cache)
        gate = ctx.beside
        if self.gate_mixer is not None:
            gate = (self.gate_mixer(h), 0)
        h = self._close(x, out, self.norms[0], gate, self.gate_bias_mixer)
        if self.ffn is not None:
            gate = self._ffn_gate(ctx, h)
            h = self._close(x, self.ffn.forward(ctx, h), self.norms[1], gate, self.gate_bias_ffn)
        ctx.beside = None
        ctx.post_rows = h
        ctx.partial_sums = False
        return x, None


def _dense(out):
    """A sub-layer's dense output as `ops.branch_step` takes it: rows, or a product still split along its k."""
    if out is None or isinstance(out, ops.Partials) or not hasattr(out, "materialize"):
        return out
    return out.materialize()
