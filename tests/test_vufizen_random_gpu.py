"""Random Vufizen configurations through the engine against the plain implementation: both mixers in any order, layers that
run again with a cache of their own, layers without feed-forward, query and key head counts, maps and values in and out of the
sizes that the matrix-core attention takes, states whose keys and values fit the chunks or not, one tap to six, maps that turn
as a whole, in part or not at all, constants of the combination from 0 up, routed experts with one expert a token up to all of
them, with and without a shared expert, widths from odd ones to those whose products run on the kernels for many rows,
vocabularies of any size.  Every configuration runs whole prompts, a prompt and then token by token, and a mixed schedule (four
live requests, pages and slots used again) in 32-bit and in bfloat16, with the measures of `test_vufizen_gpu.py` (three quantiles in bfloat16)."""
import io
import random

import numpy as np
import pytest
import torch

import plain_vufizen as pv
import trace_modes as tm
from vufizen_configs import again, attn, hgrn2, layer, model, moe, random_tokens, write_model

pytestmark = pytest.mark.gpu

LENGTHS = [1, 2, 19, 64, 150, 260]


def random_attention(rng: random.Random):
    kv = rng.choice([1, 1, 2, 3])
    dim = rng.choice([8, 16, 24, 32, 64]) if rng.random() < 0.6 else rng.choice([5, 6, 12, 20, 40])
    # (of the pairs of widths that the matrix cores take, those that are built beside the package: another pair would be
    # compiled inside the test)
    from inferrs_amd.ops.build import ATTN_HEAD_DIMS, ATTN_VALUE_PAIRS
    widths = [v for v in (8, 13, 16, 20, 32, 48, 64, 128, 256)
              if v == 2 * dim or v not in ATTN_HEAD_DIMS or 2 * dim not in ATTN_HEAD_DIMS or (2 * dim, v) in ATTN_VALUE_PAIRS]
    return attn(kv * rng.choice([1, 2, 4]), kv, dim, 2 * dim if rng.random() < 0.5 else rng.choice(widths),
                rng.choice([0.5, 1.0, 2.0]) * dim ** -0.5, conv=rng.choice([1, 2, 3, 4, 4, 6]), diff=rng.choice([0.0, 0.2, 0.5, 0.8]),
                base=rng.choice([100.0, 10000.0, 500000.0]), turned=rng.choice([dim // 2 * 2, dim // 4 * 2, 2, 0]))


def random_state(rng: random.Random):
    return hgrn2(rng.choice([1, 2, 3, 4]), rng.choice([1, 8, 10, 16, 32, 48, 100, 128, 136]), rng.choice([5, 8, 16, 32, 33, 64, 128, 160]))


def random_mlp(rng: random.Random):
    if rng.random() < 0.15:
        return None
    experts = rng.choice([1, 2, 3, 5, 8, 12, 40])
    top = min(rng.choice([1, 2, min(experts, 4), experts if experts <= 8 else 3]), experts)
    return moe(experts, top, rng.choice([8, 16, 30, 64]), shared=rng.choice([8, 24, 40, 128]) if rng.random() < 0.7 else None)


def random_config(rng: random.Random) -> dict:
    width = rng.choice([128, 256, 384]) if rng.random() < 0.4 else rng.choice([24, 33, 40, 50, 64, 72, 96])
    layers = []
    for _ in range(rng.randint(2, 5)):
        if layers and rng.random() < 0.25:
            layers.append(again(layers, rng.randrange(len(layers))))
        else:
            layers.append(layer(random_attention(rng) if rng.random() < 0.5 else random_state(rng), random_mlp(rng)))
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
    rng = random.Random(5000 + seed)
    cfg = random_config(rng)
    folder = str(tmp_path / "model")
    tensors = write_model(folder, cfg, seed=seed)
    reqs = {f"r{i}": random_tokens(n, cfg["vocab"], 70 + i) for i, n in enumerate(LENGTHS)}
    ref64 = {r: pv.forward(cfg, tensors, t).numpy() for r, t in reqs.items()}
    ref = {r: v.astype(np.float32) for r, v in ref64.items()}
    noise = {r: np.maximum.accumulate(e) for r, e in
             errors({r: pv.forward(cfg, tensors, t, dtype=torch.float32).double().numpy() for r, t in reqs.items()}, ref64, reqs).items()}
    theirs = np.concatenate(list(errors({r: pv.forward(cfg, tensors, t, dtype=torch.bfloat16).float().numpy() for r, t in reqs.items()},
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
