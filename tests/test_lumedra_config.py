"""Lumedra without a GPU: config.json -> the model as data (layers, tensor names and shapes, which layer's values are mixed
with whose, what each mixer keeps per request), the errors that name a key, and the plain implementation against itself (a
prefix, closed forms, what each mechanism is worth)."""
import copy

import pytest
import torch

import plain_lumedra as pl
from lumedra_configs import CONFIGS, attn, dense, layer, model, random_tokens, random_weights, sharpened, tensor_shapes

from inferrs_amd.cache import RELEASED, CacheManager
from inferrs_amd.config.base import ConfigError
from inferrs_amd.config.lumedra import LumedraConfig
from inferrs_amd.config.registry import resolve_architecture
from inferrs_amd.config.spec import AttentionSpec, PositionSpec, RoutedExpertsSpec, SpecError
from inferrs_amd.parts.assemble import model_tensors
from inferrs_amd.parts.attention import Attention
from inferrs_amd.parts.base import FixedState, PagedKV, part_class


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_tensor_names_and_shapes(name):
    cfg = CONFIGS[name]
    assert resolve_architecture(cfg) is LumedraConfig
    expected, optional = model_tensors(LumedraConfig.from_dict(cfg).to_spec())
    assert not optional
    assert {k: tuple(v.shape) for k, v in expected.items()} == tensor_shapes(cfg)


def test_the_model_as_data():
    spec = LumedraConfig.from_dict(CONFIGS["A"]).to_spec()
    assert [(e.layer, e.cache_of) for e in spec.schedule] == [(i, None) for i in range(6)]
    assert all(l.arrangement == "parallel" and all(n.kind == "rmsnorm" and n.eps == 1e-5 for n in l.norms) for l in spec.layers)
    assert [l.norm_names for l in spec.layers[2:4]] == [("l2.norm1", "l2.norm2"), ("l3.norm1",)]
    m = [l.mixer for l in spec.layers]
    assert [x.kind for x in m] == ["attention", "latent_attention", "lightning", "attention", "attention", "attention"]
    assert [(x.window, x.keep_first, x.softcap, x.v_mix) for x in m if x.kind == "attention"] == [
        (20, 5, 8.0, "first"), (11, 37, 3.0, None), (70, 1, 20.0, "mix"), (20, 5, None, "mix")]
    assert all(x.position.kind == "none" and not x.gate for x in m if x.kind == "attention")
    assert (m[1].q_rank, m[1].kv_rank, m[1].gate, m[1].gate_per_head, m[1].sink, m[1].window) == (20, 26, True, False, False, None)
    assert (m[1].position.pairing, m[1].position.rot_dim, m[1].position.theta) == ("interleaved", 6, 500.0)
    assert (m[2].decay, m[2].head_dim, m[2].v_dim, m[2].norm_eps) == ((0.4, 0.9, 0.998), 12, 10, 1e-5)
    f = [l.ffn for l in spec.layers]
    assert (f[0].experts, f[0].top, f[0].scale, f[0].score, f[0].renormalize, f[0].activation, f[0].groups, f[0].shared_gate) == (
        6, 2, 2.5, "sigmoid", True, "silu", (3, 2), False)
    assert f[0].shared.intermediate == 16 and f[0].shared.activation == "silu" and f[2].shared is None and f[5].groups is None
    assert (f[1].kind, f[1].limit, f[1].alpha) == ("clamped_mlp", 0.8, 1.702) and f[3] is None
    assert spec.embedding.wide and spec.head.name is None and spec.head_name is None
    assert LumedraConfig.from_dict(LumedraConfig.from_dict(CONFIGS["A"]).to_dict()).to_spec() == spec
    # windows and caps may be absent
    last = LumedraConfig.from_dict(CONFIGS["E"]).to_spec().layers[3].mixer
    assert (last.window, last.keep_first, last.softcap, last.v_mix) == (None, 0, None, "mix")


def test_what_each_mixer_keeps():
    spec = LumedraConfig.from_dict(CONFIGS["A"]).to_spec()
    needs = [part_class("mixer", l.mixer).cache_need(l.mixer) for l in spec.layers]
    assert needs == [PagedKV(2, 10, 20, v_head_dim=12, keep_first=5), PagedKV(1, 32, None), FixedState((360,)),
                     PagedKV(3, 14, 11, v_head_dim=8, keep_first=37), PagedKV(2, 16, 70, v_head_dim=12, keep_first=1),
                     PagedKV(2, 8, 20, v_head_dim=12, keep_first=5)]
    cm = CacheManager(dict(enumerate(needs)), page_size=8, num_pages=40, max_seqs=2)
    cm.add_sequence("a")
    assert cm.reserve("a", 200)
    cm.commit("a", 200)
    # 25 pages hold the latent rows; a window's group keeps the pages of its last keys (the next query's, at 200) and of its first
    held = [{i for i, p in enumerate(t) if p != RELEASED} for t in cm.sequences["a"].tables.values()]
    assert held == [{0, 22, 23, 24}, set(range(25)), {0, 1, 2, 3, 4, 23, 24}, {0} | set(range(16, 25)), {0, 22, 23, 24}]
    cm.free_sequence("a")
    cm.check_invariants()
    assert all(g.pool.num_free == 40 for g in cm.groups) and cm.slots.num_free == 2


@pytest.mark.parametrize("change, key", [
    (lambda c: c["layers"][2].__setitem__("type", "mamba2"), "layers[2].type"),
    (lambda c: c["layers"][0].pop("mixer"), "layers[0].mixer"),
    (lambda c: c["layers"][0]["mixer"].pop("scale"), "mixer.scale"),
    (lambda c: c["layers"][0]["mixer"].__setitem__("kv_heads", 3), "kv_heads"),
    (lambda c: c["layers"][0]["mixer"].__setitem__("softcap", 0.0), "mixer.softcap"),
    (lambda c: c["layers"][0]["mixer"]["mask"].pop("size"), "mask.size"),
    (lambda c: c["layers"][0]["mixer"]["mask"].__setitem__("keep_first", -1), "mask.keep_first"),
    (lambda c: c["layers"][0]["mixer"].__setitem__("mask", 5), "mixer.mask"),
    (lambda c: c["layers"][0]["mixer"].__setitem__("v_mix", 1), "mixer.v_mix"),
    (lambda c: c["layers"][4]["mixer"].__setitem__("vdim", 16), "layers[4].mixer"),
    (lambda c: c["layers"][1]["mixer"].pop("q_rank"), "mixer.q_rank"),
    (lambda c: c["layers"][1]["mixer"]["rot"].pop("base"), "rot.base"),
    (lambda c: c["layers"][1]["mixer"]["rot"].__setitem__("dims", 8), "rot.dims"),
    (lambda c: c["layers"][1]["mixer"]["rot"].__setitem__("dims", 5), "rot.dims"),
    (lambda c: c["layers"][2]["mixer"].__setitem__("decay", [0.5, 0.5]), "mixer.decay"),
    (lambda c: c["layers"][2]["mixer"].__setitem__("decay", [0.5, 0.5, 1.5]), "mixer.decay"),
    (lambda c: c["layers"][2]["mixer"].pop("vdim"), "mixer.vdim"),
    (lambda c: c["layers"][1]["mlp"].pop("limit"), "mlp.limit"),
    (lambda c: c["layers"][1]["mlp"].__setitem__("limit", 0), "mlp.limit"),
    (lambda c: c["layers"][1]["mlp"].__setitem__("kind", "gated"), "mlp.kind"),
    (lambda c: c["layers"][0]["mlp"]["router"].__setitem__("top", 5), "router.top"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].__setitem__("count", 4), "router.groups"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].__setitem__("keep", 4), "router.groups"),
    (lambda c: c["layers"][0]["mlp"]["expert"].pop("ff"), "expert.ff"),
    (lambda c: c["layers"][0]["mlp"].pop("router"), "mlp.router"),
    (lambda c: c["layers"][0]["mlp"].__setitem__("shared", 16), "mlp.shared"),
    (lambda c: c["norm"].pop("eps"), "norm.eps"),
    (lambda c: c.pop("width"), "width"),
    (lambda c: c.pop("layers"), "layers"),
])
def test_errors_name_the_key(change, key):
    cfg = copy.deepcopy(CONFIGS["A"])
    change(cfg)
    with pytest.raises(ConfigError) as e:
        LumedraConfig.from_dict(cfg)
    assert key in str(e.value)


def test_specs_that_no_kernel_honours_are_refused_by_name():
    common = dict(hidden=8, n_heads=2, n_kv_heads=1, head_dim=4, position=PositionSpec("none"))
    for bad, word in ((dict(keep_first=3), "keep_first"), (dict(window=4, softcap=-1.0), "softcap"), (dict(v_mix="last"), "v_mix"),
                      (dict(v_mix="mix", own_kv=False), "v_mix")):
        with pytest.raises(SpecError, match=word):
            Attention(AttentionSpec(**common, **bad), {}, torch.float32, "cpu")
    for bad in ((3, 1), (2, 3), (4, 1)):
        with pytest.raises(SpecError, match="groups"):
            part_class("ffn", RoutedExpertsSpec(8, 4, 8, 3))(RoutedExpertsSpec(8, 4, 8, 3, groups=bad), {}, torch.float32, "cpu")


def test_plain_against_itself():
    cfg = sharpened(CONFIGS["A"], 4.0)
    w = random_weights(cfg, 3)
    toks = random_tokens(90, cfg["vocab"], 1)
    whole = pl.forward(cfg, w, toks)
    scale = float(whole.abs().max())
    assert torch.allclose(pl.forward(cfg, w, toks[:23]), whole[:23], atol=1e-10)          # causal: a prefix gives the same logits
    streams = []
    pl.forward(cfg, w, toks, layers_out=streams)
    assert len(streams) == 6

    def moved(other_cfg=None, other_w=None):
        return float((pl.forward(other_cfg or cfg, other_w or w, toks) - whole).abs().max()) / scale

    # every mechanism is worth something
    for n in ("l0.mix.v", "l1.mix.g", "l1.mix.dkv", "l2.mix.g", "l2.mix.k", "l4.mix.vmix", "l5.mix.vmix", "l0.mlp.shared.down",
              "l2.mlp.router", "l1.mlp.up"):
        assert moved(other_w=dict(w, **{n: torch.zeros_like(w[n])})) > 1e-3, n
    for n in ("l0.norm1", "l0.norm2", "l3.norm1", "l1.mix.dq.norm", "l1.mix.dkv.norm", "l2.mix.norm", "final.norm"):
        assert moved(other_w=dict(w, **{n: torch.ones_like(w[n])})) > 1e-3, n

    def changed(i, *path_value):
        c = copy.deepcopy(cfg)
        at = c["layers"][i]
        for k in path_value[:-2]:
            at = at[k]
        at[path_value[-2]] = path_value[-1]
        return c

    for args in ((0, "mixer", "mask", "size", 21), (0, "mixer", "mask", "keep_first", 6), (0, "mixer", "mask", "keep_first", 4),
                 (3, "mixer", "mask", "keep_first", 38), (0, "mixer", "softcap", 20.0), (1, "mixer", "rot", {"base": 600.0, "dims": 6}),
                 (2, "mixer", "decay", [0.4, 0.9, 0.98]), (1, "mlp", "limit", 0.9), (0, "mlp", "router", "scale", 2.0),
                 (0, "mlp", "router", "groups", {"count": 3, "keep": 1}), (2, "mlp", "router", "groups", None),
                 (0, "mixer", "v_mix", False)):
        assert moved(changed(*args)) > 1e-3, args
    # a state carries over a cut, and its closed form
    g = torch.Generator().manual_seed(0)
    q, k, v = (torch.randn(40, 2, n, generator=g).double() for n in (6, 6, 5))
    a = (0.7, 0.95)
    o, S = pl.fading_sums(q, k, v, a)
    o1, S1 = pl.fading_sums(q[:17], k[:17], v[:17], a)
    o2, S2 = pl.fading_sums(q[17:], k[17:], v[17:], a, S1)
    assert torch.allclose(torch.cat([o1, o2]), o) and torch.allclose(S2, S)
    for h in range(2):
        closed = sum(a[h] ** (39 - s) * float(q[39, h] @ k[s, h]) * v[s, h] for s in range(40))
        assert torch.allclose(closed, o[39, h])


def test_the_mask_token_by_token():
    seen = pl.seen_keys(12, {"size": 4, "keep_first": 2})
    for i in range(12):
        assert [j for j in range(12) if seen[i, j]] == sorted(set(range(max(0, i - 3), i + 1)) | set(range(min(2, i + 1))))
    assert torch.equal(pl.seen_keys(5, None), torch.tril(torch.ones(5, 5)).bool())


def test_groups_by_hand():
    # three groups of two: the sums are 1.0, 1.1 and 0.9; of the best two groups the largest are 2, 0
    s = torch.tensor([[0.8, 0.2, 0.9, 0.2, 0.45, 0.45]])
    assert pl.best_groups(s, 3, 2).tolist() == [[True, True, True, True, False, False]]
    z = torch.log(s / (1 - s)).double()
    chosen, weight = pl.route(torch.ones(1, 1).double(), {"router": z.T}, "", {"top": 3, "scale": 2.0, "groups": {"count": 3, "keep": 2}})
    assert sorted(chosen[0].tolist()) in ([0, 1, 2], [0, 2, 3])
    assert torch.allclose(weight.sum(), torch.tensor(2.0).double()) and float(weight[0, 0]) == pytest.approx(2 * 0.9 / 1.9)


def test_a_model_of_one_layer_of_each_kind_is_read():
    cfg = model(40, 16, [layer(attn(2, 1, 8, 8, 0.3, size=4, keep_first=2, softcap=5.0), dense(16, 1.0))])
    assert LumedraConfig.from_dict(cfg).to_spec().layers[0].mixer.v_mix is None
