"""Random Lumedra configurations through the engine against the plain implementation: the three mixers in any order, query and
key head counts, heads and values in and out of the sizes that the matrix-core attention takes, latent rows likewise, windows
of one token up to longer than a request with no kept first tokens up to more than a window, caps or none, layers that mix
values and layers between them that do not, states whose keys and values fit the chunks or not with decays from 0 to 1, clamped
dense feed-forwards, routed experts with one expert a token up to all of them in one group up to as many as there are experts,
with and without a shared expert, layers without feed-forward, widths from odd ones to those whose products run on the kernels
for many rows, vocabularies of any size.  Every configuration runs whole prompts, a prompt and then token by token, and a mixed
schedule (four live requests, pages and slots used again) in 32-bit and in bfloat16, with the measures of
`test_lumedra_gpu.py` (three quantiles in bfloat16)."""
import io
import random

import numpy as np
import pytest
import torch

import plain_lumedra as pl
import trace_modes as tm
from lumedra_configs import attn, dense, latent, layer, lightning, model, moe, random_tokens, write_model

pytestmark = pytest.mark.gpu

LENGTHS = [1, 2, 19, 64, 150, 260]


def random_latent(rng: random.Random):
    dim, rot = rng.choice([8, 16, 24, 32, 13]), rng.choice([2, 4, 8, 16, 32, 6])
    rank = rng.choice([48 - rot, 64 - rot, 128 - rot, 144 - rot]) if rng.random() < 0.6 else rng.choice([12, 21, 40, 90])
    return latent(rng.choice([1, 2, 3, 6]), dim, rot, rng.choice([8, 16, 20, 48]), rng.choice([16, 24, 40, 64]), rank,
                  rng.choice([0.5, 1.0, 2.0]) * (dim + rot) ** -0.5, base=rng.choice([100.0, 10000.0, 500000.0]))


def random_attention(rng: random.Random, total: int, v_mix: bool):
    """`total`: what a token's values come to over the key heads (layers that mix share it)."""
    kv = rng.choice([k for k in (1, 2, 3) if total % k == 0])
    vdim = total // kv
    dim = vdim if rng.random() < 0.6 else rng.choice([5, 11, 20, 40, 72 + 5])      # (no pair of widths that a library would be compiled for)
    size = rng.choice([None, 1, 7, 16, 33, 64, 65, 130, 400])
    return attn(kv * rng.choice([1, 2, 4]), kv, dim, vdim, rng.choice([0.5, 1.0, 2.0]) * dim ** -0.5, size=size,
                keep_first=rng.choice([0, 1, 4, 16, 17, 40, 70]) if size is not None else 0,
                softcap=rng.choice([None, 2.0, 5.0, 30.0]), v_mix=v_mix)


def random_state(rng: random.Random):
    heads = rng.choice([1, 2, 3, 4])
    return lightning(heads, rng.choice([1, 8, 10, 16, 32, 48, 100, 128, 136]), rng.choice([5, 8, 16, 32, 33, 64, 128, 160]),
                     [rng.choice([0.0, 0.1, 0.5, 0.9, 0.99, 0.999, 1.0]) for _ in range(heads)])


def random_mlp(rng: random.Random):
    roll = rng.random()
    if roll < 0.15:
        return None
    if roll < 0.4:
        return dense(rng.choice([8, 16, 30, 64, 128]), rng.choice([0.3, 1.0, 7.0]))
    experts = rng.choice([1, 2, 4, 6, 8, 12, 40])
    count = rng.choice([c for c in (1, 2, 3, 4, experts) if experts % c == 0])
    keep = rng.randint(1, count)
    room = keep * (experts // count)
    top = min(rng.choice([1, 2, 3, room if room <= 8 else 3]), room)
    return moe(experts, top, rng.choice([8, 16, 30, 64]), rng.choice([0.5, 1.0, 2.5]), (count, keep) if rng.random() < 0.8 else None,
               shared=rng.choice([8, 24, 40, 128]) if rng.random() < 0.7 else None)


def random_config(rng: random.Random) -> dict:
    width = rng.choice([128, 256, 384]) if rng.random() < 0.4 else rng.choice([24, 33, 40, 50, 64, 72, 96])
    total = rng.choice([16, 24, 48, 64, 96, 128, 33, 30])
    layers = []
    for _ in range(rng.randint(2, 5)):
        kind = rng.choice(["latent", "lightning", "attention", "attention"])
        mixer = (random_latent(rng) if kind == "latent" else random_state(rng) if kind == "lightning"
                 else random_attention(rng, total, rng.random() < 0.7))
        layers.append(layer(mixer, random_mlp(rng)))
    return model(rng.choice([31, 64, 100, 257, 576]), width, layers, eps=rng.choice([1e-6, 1e-5]))


def run(folder, cfg, dtype, trace, out_dir):
    from inferrs_amd.engine import Engine, run_trace
    eng = Engine.from_folder(folder, dtype=dtype, page_size=16, num_pages=-(-trace.max_tokens // 16), max_seqs=4)
    run_trace(eng, trace.lines, out_dir, io.StringIO())
    eng.cache.check_invariants()
    assert not eng.cache.sequences and eng.cache.slots.num_free == eng.cache.slots.num_slots
    return trace.read(out_dir, cfg["vocab"])


def errors(got, ref, reqs):
    scale = max(float(np.abs(v).max()) for v in ref.values())
    return {r: np.array([float(np.abs(got[r][p] - ref[r][p]).max()) / scale for p in range(len(t))]) for r, t in reqs.items()}


@pytest.mark.parametrize("seed", range(24))
def test_random_configuration(tmp_path, seed):
    rng = random.Random(9000 + seed)
    cfg = random_config(rng)
    folder = str(tmp_path / "model")
    tensors = write_model(folder, cfg, seed=seed)
    reqs = {f"r{i}": random_tokens(n, cfg["vocab"], 70 + i) for i, n in enumerate(LENGTHS)}
    ref64 = {r: pl.forward(cfg, tensors, t).numpy() for r, t in reqs.items()}
    ref = {r: v.astype(np.float32) for r, v in ref64.items()}
    noise = {r: np.maximum.accumulate(e) for r, e in
             errors({r: pl.forward(cfg, tensors, t, dtype=torch.float32).double().numpy() for r, t in reqs.items()}, ref64, reqs).items()}
    theirs = np.concatenate(list(errors({r: pl.forward(cfg, tensors, t, dtype=torch.bfloat16).float().numpy() for r, t in reqs.items()},
                                        ref, reqs).values()))
    for mode, trace in (("whole", tm.whole(reqs)), ("tail", tm.prefix_then_single(reqs, 40)), ("mixed", tm.mixed(reqs, seed=seed))):
        for r, e in errors(run(folder, cfg, "float32", trace, str(tmp_path / f"{mode}_f32")), ref, reqs).items():
            assert (e <= np.maximum(2e-5, 3.0 * noise[r])).all(), \
                f"seed {seed} {mode} {r} float32: {e.max():.3g} of the scale (the plain 32-bit arithmetic: {noise[r].max():.3g}); {cfg}"
        mine = np.concatenate(list(errors(run(folder, cfg, "bfloat16", trace, str(tmp_path / f"{mode}_bf16")), ref, reqs).values()))
        assert np.isfinite(mine).all(), f"seed {seed} {mode} bfloat16: not finite; {cfg}"
        # (a close call of a router sends a request's positions apart from there on, in either arithmetic: the upper quantiles are
        # draws of few such events, the first quartile is what rounding does)
        for q, slack in ((0.25, 1.1), (0.5, 1.3), (0.9, 3.0)):
            a, b = float(np.quantile(mine, q)), float(np.quantile(theirs, q))
            assert a <= slack * b + 1e-3, f"seed {seed} {mode} bfloat16: quantile {q} of the errors {a:.3g}, plain in bfloat16 {b:.3g}; {cfg}"
