"""Configuration of the Lumedra decoder, read from its config.json.

config.json describes the model layer by layer:

    "architecture": "Lumedra", "vocab", "width", "norm": {"eps"},
    "layers": [{"type", "mixer": {...}, "mlp": {...} | null}, ...]

    type "latent_attention": heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, rot: {base, dims}
    type "lightning":        heads, dim, vdim, decay: [one a head]
    type "attention":        heads, kv_heads, dim, vdim, scale, softcap | absent, mask: {size, keep_first} | absent,
                             v_mix: true | absent
    mlp: {"kind": "dense", "ff", "limit"}
         {"kind": "moe", "router": {experts, top, scale, groups: {count, keep} | absent}, "expert": {ff}, "shared": {ff} | absent}

Every size and every constant that differs from model to model comes from there; what the design fixes stands in `to_spec`:
two RMS norms a layer, one a sub-layer, both of the stream as the layer finds it, the sub-layers' outputs added together; in
"latent_attention" neighbours paired in the turn, every earlier key, one sigmoid gate a feature; in "lightning" SiLU on
queries, keys and values, one norm over all heads, a sigmoid gate; in "attention" no turn by position, and values mixed with
those of the first layer that says `v_mix`; dense feed-forwards in the clamped form with slope 1.702; routed gated-SiLU
experts chosen by sigmoid scores, whose weights are brought to the sum `scale`, beside a shared one; logits through the
embedding table.
Tensor names: "embed", "final.norm", and for layer i "l<i>.norm1|norm2",
"l<i>.mix.dq|dq.norm|uq|dkv|dkv.norm|uk|uv|g|o", "l<i>.mix.q|k|v|g|norm|o" or "l<i>.mix.q|k|v|o|vmix",
"l<i>.mlp.gate|up|down" or "l<i>.mlp.router|e<j>.gate|up|down|shared.gate|up|down".
"""
from __future__ import annotations

import copy
from dataclasses import dataclass
from typing import Any, Dict, List, Optional, Tuple

from .base import ConfigError
from .buketar import _int, _num
from .spec import (AttentionSpec, ClampedMlpSpec, EmbeddingSpec, GatedMlpSpec, HeadSpec, LatentAttentionSpec, LayerSpec,
                   LightningSpec, ModelSpec, NormSpec, ParallelSpec, PositionSpec, RoutedExpertsSpec, ScheduleEntry)

DEFAULT_MAX_POSITION = 1 << 17
CLAMPED_SLOPE = 1.702               # a dense feed-forward's activation is g * sigmoid(1.702 g)

# tensors as the parts name them -> as the file names them
ATTENTION_NAMES = (("q_proj.weight", "q"), ("k_proj.weight", "k"), ("v_proj.weight", "v"), ("o_proj.weight", "o"), ("v_mix", "vmix"))
SHARED_NAMES = (("gate_proj.weight", "gate"), ("up_proj.weight", "up"), ("down_proj.weight", "down"))
MIXERS = ("latent_attention", "lightning", "attention")


def _object(raw: Dict[str, Any], key: str, where: str, required: bool = False) -> Optional[Dict[str, Any]]:
    v = raw.get(key)
    if v is None and not required:
        return None
    if not isinstance(v, dict):
        raise ConfigError(f"config.json: '{where}.{key}' must be an object" + ("" if required else " or absent"))
    return v


@dataclass(frozen=True)
class LumedraConfig:
    raw: Any                        # config.json as read (a dictionary), checked by `from_dict`

    architecture = "Lumedra"
    model_type = "lumedra"
    chat_template = None

    # ---- reading ----------------------------------------------------------------------------
    @classmethod
    def from_dict(cls, raw: Dict[str, Any], allow_ignored_keys: bool = False) -> "LumedraConfig":
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
    def _latent(self, where: str, m: Dict[str, Any], hidden: int, eps: float) -> LatentAttentionSpec:
        rot_dim = _int(m, "rot_dim", where, 0)
        rot = _object(m, "rot", where) or {}
        turned = _int(rot, "dims", where + ".rot", 0) if "dims" in rot else rot_dim
        if turned > rot_dim or turned % 2:
            raise ConfigError(f"config.json: '{where}.rot.dims' = {turned} must be even and within 'rot_dim' = {rot_dim}")
        position = (PositionSpec("rope", head_dim=rot_dim, rot_dim=turned, theta=_num(rot, "base", where + ".rot"), pairing="interleaved")
                    if turned else PositionSpec("none"))
        return LatentAttentionSpec(hidden=hidden, n_heads=_int(m, "heads", where), head_dim=_int(m, "dim", where), rot_dim=rot_dim,
                                   v_dim=_int(m, "vdim", where), kv_rank=_int(m, "kv_rank", where), position=position,
                                   scale=_num(m, "scale", where), norm_eps=eps, gate=True, q_rank=_int(m, "q_rank", where))

    def _lightning(self, where: str, m: Dict[str, Any], hidden: int, eps: float) -> LightningSpec:
        heads, decay = _int(m, "heads", where), m.get("decay")
        if (not isinstance(decay, list) or len(decay) != heads
                or any(isinstance(d, bool) or not isinstance(d, (int, float)) or not (0.0 <= d <= 1.0) for d in decay)):
            raise ConfigError(f"config.json: '{where}.decay' must be a list of {heads} numbers in 0..1, one a head")
        return LightningSpec(hidden=hidden, n_heads=heads, head_dim=_int(m, "dim", where), v_dim=_int(m, "vdim", where),
                             decay=tuple(float(d) for d in decay), norm_eps=eps)

    def _value_mixers(self) -> List[int]:
        """The layers that say `v_mix`, in order; the first leaves its values for the others."""
        out: List[int] = []
        for i, layer in enumerate(self.raw["layers"]):
            m = layer.get("mixer")
            if layer.get("type") == "attention" and isinstance(m, dict) and m.get("v_mix") is not None:
                if not isinstance(m["v_mix"], bool):
                    raise ConfigError(f"config.json: 'layers[{i}].mixer.v_mix' must be true or false")
                if m["v_mix"]:
                    out.append(i)
        return out

    def _attention(self, i: int, where: str, m: Dict[str, Any], hidden: int) -> AttentionSpec:
        heads, kv_heads, dim = _int(m, "heads", where), _int(m, "kv_heads", where), _int(m, "dim", where)
        vdim = _int(m, "vdim", where) if m.get("vdim") is not None else dim
        if heads % kv_heads:
            raise ConfigError(f"config.json: '{where}.heads' = {heads} is no multiple of 'kv_heads' = {kv_heads}")
        softcap = _num(m, "softcap", where) if m.get("softcap") is not None else None
        if softcap is not None and not softcap > 0.0:
            raise ConfigError(f"config.json: '{where}.softcap' = {softcap} must be positive")
        mask = _object(m, "mask", where)
        window, keep_first = None, 0
        if mask is not None:
            window = _int(mask, "size", where + ".mask")
            keep_first = _int(mask, "keep_first", where + ".mask", 0) if mask.get("keep_first") is not None else 0
        mixers, v_mix = self._value_mixers(), None
        if i in mixers:
            v_mix = "first" if i == mixers[0] else "mix"
            first = self.raw["layers"][mixers[0]]["mixer"]
            # (a token's values are mixed as the projections' rows, so the rows' width is what has to agree)
            width = first.get("kv_heads", 0) * (first.get("vdim") or first.get("dim") or 0)
            if kv_heads * vdim != width:
                raise ConfigError(f"config.json: '{where}' mixes its values, {kv_heads} heads of {vdim}, with those of layer "
                                  f"{mixers[0]}, {width} numbers a token")
        return AttentionSpec(hidden=hidden, n_heads=heads, n_kv_heads=kv_heads, head_dim=dim, position=PositionSpec("none"),
                             scale=_num(m, "scale", where), names=ATTENTION_NAMES, v_head_dim=vdim, window=window,
                             keep_first=keep_first, softcap=softcap, v_mix=v_mix)

    def _mixer(self, i: int, layer: Dict[str, Any], hidden: int, eps: float):
        kind, m, where = layer.get("type"), layer.get("mixer"), f"layers[{i}].mixer"
        if kind not in MIXERS:
            raise ConfigError(f"config.json: layers[{i}].type = {kind!r} is no mixer of this design (known: {list(MIXERS)})")
        if not isinstance(m, dict):
            raise ConfigError(f"config.json: '{where}' must be an object")
        if kind == "latent_attention":
            return self._latent(where, m, hidden, eps)
        return self._lightning(where, m, hidden, eps) if kind == "lightning" else self._attention(i, where, m, hidden)

    def _mlp(self, i: int, layer: Dict[str, Any], hidden: int):
        f, where = layer.get("mlp"), f"layers[{i}].mlp"
        if f is None:
            return None
        if not isinstance(f, dict):
            raise ConfigError(f"config.json: '{where}' must be an object or null")
        if f.get("kind") == "dense":
            limit = _num(f, "limit", where)
            if not limit > 0.0:
                raise ConfigError(f"config.json: '{where}.limit' = {limit} must be positive")
            return ClampedMlpSpec(hidden, _int(f, "ff", where), limit, CLAMPED_SLOPE)
        if f.get("kind") != "moe":
            raise ConfigError(f"config.json: '{where}.kind' = {f.get('kind')!r} is no feed-forward of this design (known: 'dense', 'moe')")
        router, expert = _object(f, "router", where, True), _object(f, "expert", where, True)
        shared = _object(f, "shared", where)
        r = where + ".router"
        experts, top = _int(router, "experts", r), _int(router, "top", r)
        groups_raw, groups, open_to = _object(router, "groups", r), None, experts
        if groups_raw is not None:
            groups = count, keep = _int(groups_raw, "count", r + ".groups"), _int(groups_raw, "keep", r + ".groups")
            if experts % count or keep > count:
                raise ConfigError(f"config.json: '{r}.groups' keeps {keep} of {count} equal groups of {experts} experts")
            open_to = keep * (experts // count)
        if top > open_to:
            raise ConfigError(f"config.json: '{r}.top' = {top} exceeds the {open_to} experts that can be chosen")
        return RoutedExpertsSpec(
            hidden=hidden, intermediate=_int(expert, "ff", where + ".expert"), experts=experts, top=top,
            scale=_num(router, "scale", r) if router.get("scale") is not None else 1.0, score="sigmoid", renormalize=True,
            activation="silu", groups=groups,
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
        norm = NormSpec(hidden, eps)
        layers = []
        for i, layer in enumerate(layers_raw):
            p, ffn = f"l{i}.", self._mlp(i, layer, hidden)
            names = (p + "norm1",) if ffn is None else (p + "norm1", p + "norm2")
            layers.append(LayerSpec(mixer=self._mixer(i, layer, hidden, eps), ffn=ffn, norms=(norm,) * len(names), norm_names=names,
                                    mixer_prefix=p + "mix.", ffn_prefix=p + "mlp.", arrangement="parallel", residual=ParallelSpec()))
        max_position = int(raw.get("max_position") or DEFAULT_MAX_POSITION)
        return ModelSpec(
            architecture=self.architecture, vocab_size=vocab, hidden=hidden, layers=tuple(layers),
            schedule=tuple(ScheduleEntry(i) for i in range(len(layers))),
            final_norm=norm, final_norm_name="final.norm", embed_name="embed", head_name=None,
            max_position=max_position, head_required=False, eos_token_ids=(),
            embedding=EmbeddingSpec(vocab, hidden, "embed", wide=True), head=HeadSpec(vocab, hidden, None, required=False))
