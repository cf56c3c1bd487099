"""Vufizen without a GPU: config.json -> the model as data (layers, run order, which layer's tensors a stop uses, tensor names
and shapes, what each mixer keeps per request), the errors that name a key, and the plain implementation against itself (a
prefix, what each mechanism is worth)."""
import copy

import pytest
import torch

import plain_vufizen as pv
from vufizen_configs import CONFIGS, random_tokens, random_weights, sharpened, tensor_shapes

from inferrs_amd.cache import CacheManager
from inferrs_amd.config.base import ConfigError
from inferrs_amd.config.registry import resolve_architecture
from inferrs_amd.config.vufizen import VufizenConfig
from inferrs_amd.parts.assemble import model_tensors
from inferrs_amd.parts.base import FixedState, PagedAndState, PagedKV, part_class


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_tensor_names_and_shapes(name):
    cfg = CONFIGS[name]
    assert resolve_architecture(cfg) is VufizenConfig
    spec = VufizenConfig.from_dict(cfg).to_spec()
    expected, optional = model_tensors(spec)
    assert optional == {"head"}           # (a file without it would take its logits through the embedding's table)
    assert {k: tuple(v.shape) for k, v in expected.items()} == tensor_shapes(cfg)


def test_the_model_as_data():
    spec = VufizenConfig.from_dict(CONFIGS["A"]).to_spec()
    # layers 3, 4 and 5 have no tensors: stops of their own (each with a cache of its own) that run layers 1, 0 and 1
    assert [(e.layer, e.cache_of) for e in spec.schedule] == [(0, None), (1, None), (2, None), (1, None), (0, None), (1, None)]
    assert len(spec.layers) == 3
    assert all(l.arrangement == "gated_branch" and all(n.scalar and n.kind == "rmsnorm" for n in l.norms) for l in spec.layers)
    assert [l.residual.gate_names for l in spec.layers] == [("l0.rg1", "l0.rg2"), ("l1.rg1", "l1.rg2"), ("l2.rg1",)]
    m0, m1 = spec.layers[0].mixer, spec.layers[1].mixer
    assert (m0.kind, m0.n_heads, m0.n_kv_heads, m0.head_dim, m0.v_dim, m0.conv, m0.diff) == ("differential_attention", 4, 2, 8, 12, 4, 0.3)
    assert m0.position.pairing == "interleaved" and m0.position.rot_dim == 6 and m0.position.theta == 500.0
    assert (m1.kind, m1.n_heads, m1.head_dim, m1.v_dim, m1.norm_eps) == ("hgrn2", 3, 12, 10, 1e-5)
    f0, f1 = spec.layers[0].ffn, spec.layers[1].ffn
    assert (f0.experts, f0.top, f0.score, f0.renormalize, f0.activation, f0.shared_gate) == (5, 2, "softmax", True, "silu", True)
    assert f0.shared.intermediate == 16 and f0.shared.activation == "silu" and f1.shared is None and not f1.shared_gate
    assert spec.layers[2].ffn is None and spec.final_norm.scalar and spec.embedding.wide
    assert VufizenConfig.from_dict(CONFIGS["B"]).to_spec().layers[0].mixer.position.kind == "none"
    assert VufizenConfig.from_dict(VufizenConfig.from_dict(CONFIGS["A"]).to_dict()).to_spec() == spec


def test_what_each_mixer_keeps():
    spec = VufizenConfig.from_dict(CONFIGS["A"]).to_spec()
    needs = [part_class("mixer", spec.layers[e.layer].mixer).cache_need(spec.layers[e.layer].mixer) for e in spec.schedule]
    # attention: keys of two maps and values in pages, the last three inputs of 2 * 4 * 8 + 2 * 2 * 8 + 2 * 12 channels
    first = PagedAndState(PagedKV(2, 16, None, v_head_dim=12), FixedState((3 * 120,)))
    state = FixedState((3 * 12 * 10,))
    assert needs == [first, state, PagedAndState(PagedKV(1, 24, None, v_head_dim=8), FixedState((80,))), state, first, state]
    one = VufizenConfig.from_dict(CONFIGS["B"]).to_spec().layers[0].mixer
    assert part_class("mixer", one).cache_need(one) == PagedKV(1, 128, None, v_head_dim=64)        # (one tap needs no inputs kept)
    cm = CacheManager(dict(enumerate(needs)), page_size=8, num_pages=40, max_seqs=2)
    cm.add_sequence("a")
    assert cm.reserve("a", 200)
    cm.commit("a", 200)
    assert all(g.pool.num_free == 40 - 25 for g in cm.groups) and cm.slots.num_free == 1
    cm.free_sequence("a")
    cm.check_invariants()
    assert all(g.pool.num_free == 40 for g in cm.groups) and cm.slots.num_free == 2


@pytest.mark.parametrize("change, key", [
    (lambda c: c["layers"][2].__setitem__("type", "mamba2"), "layers[2].type"),
    (lambda c: c["layers"][3].__setitem__("weights_of", 9), "weights_of"),
    (lambda c: c["layers"][3].__setitem__("weights_of", 3), "weights_of"),
    (lambda c: c["layers"][3].__setitem__("weights_of", 0), "layers[3]"),
    (lambda c: c["layers"][4]["mixer"].__setitem__("scale", 0.5), "layers[4].mixer"),
    (lambda c: c["layers"][0]["mixer"].pop("scale"), "mixer.scale"),
    (lambda c: c["layers"][0]["mixer"].pop("diff"), "mixer.diff"),
    (lambda c: c["layers"][2]["mixer"].pop("conv"), "mixer.conv"),
    (lambda c: c["layers"][2]["mixer"]["rot"].__setitem__("dims", 7), "rot.dims"),
    (lambda c: c["layers"][2]["mixer"]["rot"].__setitem__("dims", 14), "rot.dims"),
    (lambda c: c["layers"][2]["mixer"]["rot"].pop("base"), "rot.base"),
    (lambda c: c["layers"][2]["mixer"].__setitem__("kv_heads", 3), "kv_heads"),
    (lambda c: c["layers"][1]["mixer"].pop("vdim"), "mixer.vdim"),
    (lambda c: c["layers"][1].pop("mixer"), "layers[1].mixer"),
    (lambda c: c["layers"][2].__setitem__("mlp", {"kind": "dense", "ff": 8}), "mlp.kind"),
    (lambda c: c["layers"][2].__setitem__("mlp", {"kind": "moe", "router": {"experts": 2, "top": 3}, "expert": {"ff": 8}}), "router.top"),
    (lambda c: c["layers"][2].__setitem__("mlp", {"kind": "moe", "router": {"experts": 2, "top": 1}, "expert": {}}), "expert.ff"),
    (lambda c: c["norm"].pop("eps"), "norm.eps"),
    (lambda c: c.pop("width"), "width"),
])
def test_errors_name_the_key(change, key):
    cfg = copy.deepcopy(CONFIGS["A"])
    change(cfg)
    with pytest.raises(ConfigError) as e:
        VufizenConfig.from_dict(cfg)
    assert key in str(e.value)


def test_plain_against_itself():
    cfg = sharpened(CONFIGS["A"], 4.0)
    w = random_weights(cfg, 3)
    toks = random_tokens(70, cfg["vocab"], 1)
    whole = pv.forward(cfg, w, toks)
    scale = float(whole.abs().max())
    assert torch.allclose(pv.forward(cfg, w, toks[:23]), whole[:23], atol=1e-10)          # causal: a prefix gives the same logits
    streams = []
    pv.forward(cfg, w, toks, layers_out=streams)
    assert len(streams) == 6

    def moved(other_cfg=None, other_w=None):
        return float((pv.forward(other_cfg or cfg, other_w or w, toks) - whole).abs().max()) / scale

    # every mechanism is worth something: lambda's learned part and its constant, the convolution's oldest tap, the norms, the
    # turn, the gates' floor and bias, the branch gates and their biases, the shared expert and its gate
    for n in ("l0.mix.lq1", "l2.mix.lk2", "l1.mix.lower", "l1.mix.f.b", "l0.rg1", "l0.rg1.b", "l1.rg2", "l1.rg2.b", "l0.mlp.shared.sg",
              "l0.mlp.shared.down", "l1.mlp.router"):
        assert moved(other_w=dict(w, **{n: torch.zeros_like(w[n])})) > 1e-3, n
    for n in ("l0.mix.q.norm", "l2.mix.k.norm", "l1.mix.norm", "l0.norm1", "l1.norm2", "final.norm"):
        assert moved(other_w=dict(w, **{n: torch.ones_like(w[n])})) > 1e-3, n
    for n in ("l0.mix.q.conv", "l0.mix.k.conv", "l0.mix.v.conv"):
        t = w[n].clone()
        t[:, 0] = 0
        assert moved(other_w=dict(w, **{n: t})) > 1e-3, n
    for key, value in (("diff", 0.31), ("rot", {"base": 500.0, "dims": 4}), ("rot", {"base": 600.0, "dims": 6})):
        c = copy.deepcopy(cfg)
        c["layers"][0]["mixer"][key] = value
        c["layers"][4]["mixer"][key] = value
        assert moved(c) > 1e-3, key
    c = copy.deepcopy(cfg)
    c["layers"].pop()                                       # (the second run of a layer is a layer of its own)
    assert moved(c) > 1e-3
    # the two maps are two softmaxes; a state of the recurrence carries over a cut
    g = torch.Generator().manual_seed(0)
    q, v = torch.randn(40, 2, 6, generator=g).double(), torch.randn(40, 2, 5, generator=g).double()
    f = torch.rand(40, 2, 6, generator=g).double()
    o, S = pv.fading_outer_products(q, f, v)
    o1, S1 = pv.fading_outer_products(q[:17], f[:17], v[:17])
    o2, S2 = pv.fading_outer_products(q[17:], f[17:], v[17:], S1)
    assert torch.allclose(torch.cat([o1, o2]), o) and torch.allclose(S2, S)
    closed = torch.einsum("hi,hij->hj", q[39], torch.stack([(torch.prod(f[s + 1:], 0) * (1 - f[s]))[:, :, None] * v[s][:, None, :]
                                                            for s in range(40)]).sum(0))
    assert torch.allclose(closed, o[39])
