"""Configuration of the Vufizen decoder, read from its config.json.

config.json describes the model layer by layer:

    "architecture": "Vufizen", "vocab", "width", "norm": {"eps"},
    "layers": [{"type", "mixer": {...}, "mlp": {...} | null, "weights_of": j (optional)}, ...]

    type "attention": heads, kv_heads, dim, vdim, scale, diff, conv (taps), rot: {base, dims}
    type "hgrn2":     heads, dim, vdim
    mlp: {"kind": "moe", "router": {experts, top}, "expert": {ff}, "shared": {ff} | absent}

A layer with "weights_of" has no tensors of its own: it runs layer j's mixer, feed-forward and norms once more, with a cache
or state of its own (a second stop of the schedule that names the same layer).  Every size and every constant that differs
from model to model comes from config.json; what the design fixes stands in `to_spec`: sub-layers that read the stream as it
stands, a sigmoid gate a feature and an RMS norm with one number behind each; in "attention" two maps a head, a per-map
norm, neighbours paired in the turn; routed gated-SiLU experts weighted by a softmax over the chosen logits, a shared one
behind a sigmoid gate a token; logits through a matrix of their own.
Tensor names: "embed", "final.norm", "head", and for layer i "l<i>.norm1|norm2", "l<i>.rg1|rg2 (+ .b)",
"l<i>.mix.q|k|v (+ .conv)|q.norm|k.norm|lq1|lk1|lq2|lk2|o" or "l<i>.mix.q|f|f.b|lower|v|norm|o",
"l<i>.mlp.router|e<j>.gate|up|down|shared.gate|up|down|sg".
"""
from __future__ import annotations

import copy
from dataclasses import dataclass
from typing import Any, Dict, List, Tuple

from .base import ConfigError
from .buketar import _int, _num
from .spec import (DifferentialAttentionSpec, EmbeddingSpec, FadingStateSpec, GatedBranchSpec, GatedMlpSpec, LayerSpec, ModelSpec,
                   NormSpec, PositionSpec, RoutedExpertsSpec, ScheduleEntry)

DEFAULT_MAX_POSITION = 1 << 17

# the shared expert's tensors as the feed-forward part names them -> as the file names them
SHARED_NAMES = (("gate_proj.weight", "gate"), ("up_proj.weight", "up"), ("down_proj.weight", "down"))
MIXERS = ("attention", "hgrn2")


@dataclass(frozen=True)
class VufizenConfig:
    raw: Any                        # config.json as read (a dictionary), checked by `from_dict`

    architecture = "Vufizen"
    model_type = "vufizen"
    chat_template = None

    # ---- reading ----------------------------------------------------------------------------
    @classmethod
    def from_dict(cls, raw: Dict[str, Any], allow_ignored_keys: bool = False) -> "VufizenConfig":
        cfg = cls(copy.deepcopy(raw))
        cfg.to_spec()                # every key is read and checked there
        return cfg

    def to_dict(self) -> Dict[str, Any]:
        out = copy.deepcopy(self.raw)
        out.setdefault("architecture", self.architecture)
        return out

    @property
    def vocab_size(self) -> int:
        return _int(self.raw, "vocab", "")

    @property
    def hidden_size(self) -> int:
        return _int(self.raw, "width", "")

    @property
    def eos_token_ids(self) -> Tuple[int, ...]:
        return ()

    # ---- the model as data --------------------------------------------------------------------
    def owners(self) -> List[int]:
        """For every layer of config.json the layer whose tensors it uses (itself unless it says `weights_of`)."""
        layers = self.raw["layers"]
        out: List[int] = []
        for i in range(len(layers)):
            j, seen = i, {i}
            while layers[j].get("weights_of") is not None:
                where = f"layers[{j}]"
                k = _int(layers[j], "weights_of", where, 0)
                if k >= len(layers) or k in seen:
                    raise ConfigError(f"config.json: '{where}.weights_of' = {k} must lead to a layer with tensors of its own")
                seen.add(k)
                j = k
            out.append(j)
        return out

    def _attention(self, i: int, m: Dict[str, Any], hidden: int, eps: float) -> DifferentialAttentionSpec:
        where = f"layers[{i}].mixer"
        dim = _int(m, "dim", where)
        vdim = _int(m, "vdim", where) if m.get("vdim") is not None else dim
        heads, kv_heads = _int(m, "heads", where), _int(m, "kv_heads", where)
        if heads % kv_heads:
            raise ConfigError(f"config.json: '{where}.heads' = {heads} is no multiple of 'kv_heads' = {kv_heads}")
        rot = m.get("rot")
        if rot is not None and not isinstance(rot, dict):
            raise ConfigError(f"config.json: '{where}.rot' must be an object or absent")
        turned = _int(rot, "dims", where + ".rot", 0) if rot else 0
        if turned > dim or turned % 2:
            raise ConfigError(f"config.json: '{where}.rot.dims' = {turned} must be even and within {dim}")
        position = (PositionSpec("rope", head_dim=dim, rot_dim=turned, theta=_num(rot, "base", where + ".rot"), pairing="interleaved")
                    if turned else PositionSpec("none"))
        return DifferentialAttentionSpec(hidden=hidden, n_heads=heads, n_kv_heads=kv_heads, head_dim=dim, v_dim=vdim,
                                         position=position, scale=_num(m, "scale", where), diff=_num(m, "diff", where),
                                         conv=_int(m, "conv", where), norm_eps=eps)

    def _mixer(self, i: int, layer: Dict[str, Any], hidden: int, eps: float):
        kind, m = layer.get("type"), layer.get("mixer")
        if kind not in MIXERS:
            raise ConfigError(f"config.json: layers[{i}].type = {kind!r} is no mixer of this design (known: {list(MIXERS)})")
        where = f"layers[{i}].mixer"
        if not isinstance(m, dict):
            raise ConfigError(f"config.json: '{where}' must be an object")
        if kind == "attention":
            return self._attention(i, m, hidden, eps)
        return FadingStateSpec(hidden=hidden, n_heads=_int(m, "heads", where), head_dim=_int(m, "dim", where),
                               v_dim=_int(m, "vdim", where), norm_eps=eps)

    def _mlp(self, i: int, layer: Dict[str, Any], hidden: int):
        f = layer.get("mlp")
        if f is None:
            return None
        where = f"layers[{i}].mlp"
        if not isinstance(f, dict) or f.get("kind") != "moe":
            raise ConfigError(f"config.json: '{where}.kind' is no feed-forward of this design (known: 'moe')")
        expert, router, shared = f.get("expert"), f.get("router"), f.get("shared")
        if not isinstance(expert, dict) or not isinstance(router, dict):
            raise ConfigError(f"config.json: '{where}' needs the objects 'router' and 'expert'")
        experts, top = _int(router, "experts", where + ".router"), _int(router, "top", where + ".router")
        if top > experts:
            raise ConfigError(f"config.json: '{where}.router.top' = {top} exceeds the router's {experts} experts")
        if shared is not None and not isinstance(shared, dict):
            raise ConfigError(f"config.json: '{where}.shared' must be an object or null")
        # (a softmax over all logits, renormalised over the chosen ones, is the softmax over the chosen ones)
        return RoutedExpertsSpec(
            hidden=hidden, intermediate=_int(expert, "ff", where + ".expert"), experts=experts, top=top, score="softmax",
            renormalize=True, activation="silu", shared_gate=shared is not None,
            shared=None if shared is None else GatedMlpSpec(hidden, _int(shared, "ff", where + ".shared"), names=SHARED_NAMES))

    def to_spec(self) -> ModelSpec:
        raw = self.raw
        if not isinstance(raw, dict):
            raise ConfigError("config.json must hold an object")
        vocab, hidden = self.vocab_size, self.hidden_size
        eps = _num(raw.get("norm"), "eps", "norm")
        layers_raw = raw.get("layers")
        if not isinstance(layers_raw, list) or not layers_raw:
            raise ConfigError("config.json: 'layers' must be a list with at least one layer")
        for i, layer in enumerate(layers_raw):
            if not isinstance(layer, dict):
                raise ConfigError(f"config.json: layers[{i}] must be an object")
        owners = self.owners()
        norm = NormSpec(hidden, eps, scalar=True)
        layers, place = [], {}
        for i, layer in enumerate(layers_raw):
            if owners[i] != i:
                continue
            p, ffn = f"l{i}.", self._mlp(i, layer, hidden)
            branches = ("1",) if ffn is None else ("1", "2")
            place[i] = len(layers)
            layers.append(LayerSpec(mixer=self._mixer(i, layer, hidden, eps), ffn=ffn, norms=(norm,) * len(branches),
                                    norm_names=tuple(p + "norm" + b for b in branches), mixer_prefix=p + "mix.", ffn_prefix=p + "mlp.",
                                    arrangement="gated_branch", residual=GatedBranchSpec(tuple(p + "rg" + b for b in branches))))
        for i, j in enumerate(owners):
            for key in ("type", "mixer", "mlp"):
                if layers_raw[i].get(key) != layers_raw[j].get(key):
                    raise ConfigError(f"config.json: 'layers[{i}].{key}' differs from layer {j}'s, whose tensors it uses")
        max_position = int(raw.get("max_position") or DEFAULT_MAX_POSITION)
        return ModelSpec(
            architecture=self.architecture, vocab_size=vocab, hidden=hidden, layers=tuple(layers),
            schedule=tuple(ScheduleEntry(place[j]) for j in owners),
            final_norm=norm, final_norm_name="final.norm", embed_name="embed", head_name="head",
            max_position=max_position, head_required=True, eos_token_ids=(),
            embedding=EmbeddingSpec(vocab, hidden, "embed", wide=True))
