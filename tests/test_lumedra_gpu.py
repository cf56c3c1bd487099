"""Lumedra on the GPU against the plain implementation (`plain_lumedra.py`, 64-bit).

Mechanisms alone, through the kernels' Python face: two norms of one stream out of the kernel between layers; values mixed on
their way to the cache; attention over a window beside the first few keys, with and without capped scores, in every attention
kernel (keys that stand out just inside and just outside every edge, far away and at page borders, pages that were given back
holding NaN, any split of the keys); lightning attention's recurrence in its walk and in its chunks (portions cut anywhere,
decays from 0 to 1, a key read hundreds of tokens later, slots used again) with the norm over all heads behind it; the choice
of experts inside the best groups; latent attention with a gate a feature.  Then whole models through the engine's step function
under every way of cutting the work (whole prompts, a prompt and then token by token, every token alone, portions down to two
tokens, up to four live requests mixed in a pool whose pages and slots are used again), in both precisions, with ordinary
weights and with sharpened queries.  Greedy generation runs through the engine's own entry point and scheduler, the command
line and the replay program.

Tolerances.  32-bit: 2e-5 of the largest logit against the 64-bit result, at every position; where the plain
implementation's own 32-bit arithmetic is further off than a third of that up to there, three times what it is off.  bfloat16:
the measure is the distribution of the positions' errors against that of the plain implementation in bfloat16 arithmetic
(every operation rounded) on the same positions: the engine keeps more in 32-bit than that, so its median and its ninth
decile must not be larger (a tenth and a half of slack)."""
import io
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import plain_lumedra as pl
import trace_modes as tm
from lumedra_configs import CONFIGS, random_tokens, sharpened, write_model

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
LENGTHS = [1, 2, 3, 17, 64, 65, 130, 300, 700]
TOL_F32 = 2e-5
CASES = [("A", 1.0), ("B", 1.0), ("C", 1.0), ("D", 1.0), ("E", 1.0), ("F", 1.0), ("A", 4.0), ("D", 2.5)]
BOTH = pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])


def dev(t, dtype=None):
    return t.to(device="cuda", dtype=dtype or t.dtype).contiguous()


def i32(*v):
    return dev(torch.tensor(v, dtype=torch.int32))


def assert_close(got, want, rel, what):
    err = float((got.double().cpu() - want).abs().max()) / max(float(want.abs().max()), 1e-9)
    assert err <= rel, f"{what}: {err:.3g} of the scale, allowed {rel:.3g}"


# ---- two norms of one stream -------------------------------------------------------------------------------

@pytest.mark.parametrize("W", [40, 33, 304, 5000, 9000])
@BOTH
def test_two_norms_of_one_stream(W, dtype):
    from inferrs_amd import ops
    g = torch.Generator().manual_seed(W)
    n, top = 13, 3
    x = 3 * torch.randn(n, W, generator=g) + 0.7
    y1, y3 = (torch.randn(n, W, generator=g).to(dtype) for _ in range(2))
    routed, rw = torch.randn(n, top, W, generator=g), torch.rand(n, top, generator=g)
    w1, w2, b1, b2 = (0.5 + torch.rand(W, generator=g) for _ in range(4))
    rel = 5e-3 if dtype == torch.bfloat16 else 3e-6
    want = x.double() + y1.double() + (rw.double()[:, :, None] * routed.double()).sum(1) + y3.double()
    xs = dev(x)
    _, (h1, h2) = ops.parallel_step(xs, y1=dev(y1), routed=dev(routed), routed_weights=dev(rw), y3=dev(y3), norm_weight=dev(w1),
                                    norm2_weight=dev(w2), norm_eps=1e-5, center=False, h_dtype=dtype)
    assert_close(xs, want, 2e-6, "the sum")
    assert_close(h1, pl.rms_norm(want, w1.double(), 1e-5), rel, "the first norm")
    assert_close(h2, pl.rms_norm(want, w2.double(), 1e-5), rel, "the second norm")
    # the first is what it is without a second; layer norms, each with its own bias; a product still split along its k
    xs = dev(x)
    _, one = ops.parallel_step(xs, y1=dev(y1), routed=dev(routed), routed_weights=dev(rw), y3=dev(y3), norm_weight=dev(w1),
                               norm_eps=1e-5, center=False, h_dtype=dtype)
    assert torch.equal(one, h1)
    parts = torch.randn(3, n, W, generator=g)
    xs = dev(x)
    _, (h1, h2) = ops.parallel_step(xs, y1=ops.Partials(dev(parts)), norm_weight=dev(w1), norm_bias=dev(b1), norm2_weight=dev(w2),
                                    norm2_bias=dev(b2), norm_eps=1e-5, center=True, h_dtype=dtype)
    want = x.double() + parts.double().sum(0)
    unit = (want - want.mean(-1, keepdim=True)) / torch.sqrt(want.var(-1, unbiased=False, keepdim=True) + 1e-5)
    assert_close(h1, unit * w1.double() + b1.double(), rel, "the first layer norm")
    assert_close(h2, unit * w2.double() + b2.double(), rel, "the second layer norm")


# ---- values mixed on their way to the cache ------------------------------------------------------------------

@pytest.mark.parametrize("H,G,d,dv", [(4, 2, 10, 12), (6, 3, 64, 64), (2, 1, 48, 24), (4, 4, 11, 13), (8, 2, 128, 64)])
@BOTH
def test_mixed_values(H, G, d, dv, dtype):
    from inferrs_amd import ops
    g = torch.Generator().manual_seed(d + dv)
    n, page = 37, 8
    ld = H * d + G * d + G * dv + 8
    rows, other = torch.randn(n, ld, generator=g).to(dtype), torch.randn(n, ld, generator=g).to(dtype)
    at = H * d + G * d
    pages = -(-n // page)
    perm = torch.randperm(pages, generator=g)
    pos = torch.arange(n)
    slots = (perm[pos // page] * page + pos % page).to(torch.int32)
    for mix in (0.0, 0.37, 1.0, -0.4):
        kc, vc = (dev(torch.full(s, float("nan"), dtype=dtype)) for s in ((pages, G, page, d), (pages, G, dv, page)))
        q = ops.qk_rope_kv_strided(dev(rows), H, G, d, dv, q_off=0, k_off=H * d, v_off=at, q_norm_w=None, k_norm_w=None, eps=0.0,
                                   add_one=False, cos=None, sin=None, rot=0, interleaved=False, k_cache=kc, v_cache=vc, slots=dev(slots),
                                   page_size=page, v_with=dev(other)[:, at:at + G * dv], v_mix=mix)
        assert torch.equal(q.cpu().view(n, H * d), rows[:, :H * d])
        assert torch.equal(kc.cpu()[perm[pos // page], :, pos % page].view(n, G * d), rows[:, H * d:at])
        want = pl.mixed_values(rows[:, at:at + G * dv].double(), other[:, at:at + G * dv].double(), mix)
        assert_close(vc.cpu()[perm[pos // page], :, :, pos % page].reshape(n, G * dv), want, 4e-3 if dtype == torch.bfloat16 else 1e-6, f"mix {mix}")


# ---- attention over a window beside the first keys, capped scores ---------------------------------------------------

MASKS = [(4, 2, 8, 12, 150, 20, 5, 3.0), (4, 2, 128, 128, 700, 100, 70, 4.0), (4, 2, 128, 128, 500, 65, 64, None), (8, 1, 128, 64, 400, 129, 1, 5.0),
         (6, 2, 48, 48, 300, 33, 6, 3.0), (4, 4, 64, 64, 330, 64, 130, None), (3, 3, 11, 13, 90, 6, 19, 2.0), (16, 2, 64, 64, 260, 1, 0, 3.0),
         (4, 2, 128, 128, 300, None, 0, 3.0), (20, 1, 32, 32, 200, 40, 16, None), (4, 2, 24, 40, 700, 600, 3, 8.0), (2, 1, 16, 16, 140, 100, 200, 2.0),
         (4, 1, 144, 144, 300, 90, 33, 6.0)]


class Step:
    pass


def mask_case(H, G, d, dv, n, size, keep, cap, dtype):
    """Rows of q, k, v with keys that stand out just inside and just outside every edge of some queries' windows, and the plain result."""
    g = torch.Generator().manual_seed(n + d)
    q, k, v = torch.randn(n, H, d, generator=g), torch.randn(n, G, d, generator=g), torch.randn(n, G, dv, generator=g)
    mask = {"size": size, "keep_first": keep} if size is not None else None
    seen = pl.seen_keys(n, mask)
    planted = []
    for i in sorted({n - 1, n - 2, n // 2, n // 2 + 1, 3 * n // 4, min(n - 1, (size or n) + keep + 40)}):
        for j in (0, keep - 1, keep, keep + 1, 15, 16, 63, 64, i - (size or n), i - (size or n) + 1, i, i // 16 * 16 - 1, i // 64 * 64):
            if 0 <= j <= i:
                planted.append((i, j))
    for i, j in planted:                             # (the last to be planted wins a key)
        k[j, 0] = 2.0 * q[i, 0] / q[i, 0].norm() * d ** 0.5
    scale = 2.0 * d ** -0.5
    q, k, v = q.to(dtype), k.to(dtype), v.to(dtype)
    want = pl.grouped_attention(q.double(), k.double(), v.double(), scale, cap, seen)
    shown = sum(1 for i, j in planted if seen[i, j]), sum(1 for i, j in planted if not seen[i, j])
    return q, k, v, seen, planted, shown, scale, want


@pytest.mark.parametrize("case", MASKS, ids=lambda c: "-".join(str(x) for x in c))
@BOTH
def test_window_first_keys_and_caps(case, dtype):
    from inferrs_amd import ops
    from inferrs_amd.config.spec import AttentionSpec, PositionSpec
    from inferrs_amd.parts.attention import Attention
    H, G, d, dv, n, size, keep, cap = case
    q, k, v, seen, planted, shown, scale, want = mask_case(*case, dtype)
    if size is not None:
        assert shown[0] > 3 and (shown[1] > 3 or keep > size)
        # (what is hidden would be worth something if it were seen, and what is seen if it were hidden)
        for other in ({"size": size + 1, "keep_first": keep}, {"size": size, "keep_first": keep + 1}, {"size": max(size - 1, 1), "keep_first": max(keep - 1, 0)}):
            if size + keep < n and not torch.equal(pl.seen_keys(n, other), seen):
                off = pl.grouped_attention(q.double(), k.double(), v.double(), scale, cap, pl.seen_keys(n, other))
                assert float((off - want).abs().max()) > 0.05 * float(want.abs().max()), other
    spec = AttentionSpec(hidden=8, n_heads=H, n_kv_heads=G, head_dim=d, position=PositionSpec("none"), scale=scale, v_head_dim=dv, window=size,
                         keep_first=keep if size is not None else 0, softcap=cap)
    g = torch.Generator().manual_seed(1)
    rel = 3e-2 if dtype == torch.bfloat16 else 2e-5
    for page in ((16, 32) if n < 400 else (16,)):
        pages = -(-n // page)
        perm = 1 + torch.randperm(pages, generator=g)                        # page 0 holds NaN: what a page that was given back names
        kept = -(-keep // page)
        for portions in ([n], [n - 40] + [1] * 40, [33, 2, 100, 5, 64]):
            kc, vc = (dev(torch.full(s, float("nan"), dtype=dtype)) for s in ((pages + 1, G, page, d), (pages + 1, G, dv, page)))
            at, i = 0, 0
            while at < n:
                q_len = min(portions[i % len(portions)], n - at)
                i += 1
                pos = torch.arange(at, at + q_len)
                slot_page, slot = perm[pos // page], pos % page
                kc[slot_page, :, slot] = dev(k[at:at + q_len])
                vc[slot_page, :, :, slot] = dev(v[at:at + q_len])
                ctx, group, cache = Step(), Step(), Step()
                ctx.positions, ctx.token_seq, ctx.cu_tokens = dev(pos.to(torch.int32)), dev(torch.zeros(q_len, dtype=torch.int32)), i32(0, q_len)
                ctx.n_single, ctx.n_seqs, ctx.n_tokens, ctx.max_q_len, ctx.max_kv_len = int(q_len == 1), 1, q_len, q_len, at + q_len
                ctx.max_kv_single = ctx.max_kv_multi = at + q_len
                table = perm.clone()
                if size is not None:
                    table[kept:max(kept, max(0, at - size + 1) // page)] = 0
                group.page_size, group.block_table = page, dev(table.to(torch.int32)[None, :].contiguous())
                cache.k, cache.v = kc, vc
                got = Attention.attend(spec, ctx, dev(q[at:at + q_len]), cache, group)
                assert_close(got, want[at:at + q_len], rel, f"page {page}, portions {portions[:3]} at {at}")
                at += q_len
    # any split of the keys, portions and single tokens alike
    if ops.attention_mfma_fits(dtype, d, page, dv):
        table = dev(perm.to(torch.int32)[None, :].contiguous())
        for start in (0, n - 1):
            for splits in (1, 2, 3, 5):
                got = ops.attention_mfma(dev(q[start:]), kc, vc, dev(torch.arange(start, n, dtype=torch.int32)), i32(0, n - start), table,
                                         max_q_len=n - start, max_kv_len=n, window=size, scale=scale, splits=splits,
                                         keep_first=spec.keep_first, softcap=cap)
                assert_close(got, want[start:], rel, f"{splits} splits from {start}")
    elif size is not None and n > 512 and dtype == torch.float32:
        # the plain kernel: a wave a segment, and a wave that walks them all, the same bits
        few = dict(window=size, scale=scale, max_kv_len=n, keep_first=keep, softcap=cap)
        args = (dev(q[-3:]), kc, vc, dev(torch.arange(n - 3, n, dtype=torch.int32)), dev(torch.zeros(3, dtype=torch.int32)),
                dev(perm.to(torch.int32)[None, :].contiguous()))
        assert torch.equal(ops.attention_generic(*args, split=True, **few), ops.attention_generic(*args, split=False, **few))


@pytest.mark.parametrize("tiles", [0, 2, 3])
def test_first_keys_in_every_shape_of_the_portions_kernel(tiles):
    """Blocks of 64 and of 128 columns and single waves, whatever the step's size would pick."""
    from inferrs_amd import ops
    H, G, d, n = 4, 2, 128, 700
    lib = ops.library(ops._build.attn_target(d))
    for size, keep, cap in ((100, 70, 4.0), (64, 64, None), (190, 3, 2.0), (33, 300, 3.0)):
        q, k, v, seen, planted, shown, scale, want = mask_case(H, G, d, d, n, size, keep, cap, torch.bfloat16)
        page, pages = 16, -(-n // 16)
        kc = dev(k.view(-1, 1)[:0].new_zeros(pages, G, page, d))
        vc = dev(v.new_zeros(pages, G, d, page))
        pos = torch.arange(n)
        kc[pos // page, :, pos % page] = dev(k)
        vc[pos // page, :, :, pos % page] = dev(v)
        table = dev(torch.arange(pages, dtype=torch.int32)[None, :].contiguous())
        try:
            lib.ia_attention_mfma_tiles(tiles)
            for start in (0, 130, 517):
                for splits in (1, 3):
                    got = ops.attention_mfma(dev(q[start:]), kc, vc, dev(torch.arange(start, n, dtype=torch.int32)), i32(0, n - start), table,
                                             max_q_len=n - start, max_kv_len=n, window=size, scale=scale, splits=splits, keep_first=keep, softcap=cap)
                    assert_close(got, want[start:], 3e-2, f"window {size}, first {keep}, from {start}, {splits} splits")
        finally:
            lib.ia_attention_mfma_tiles(1)


# ---- lightning attention ---------------------------------------------------------------------------------------

def cut_steps(lengths, portions, seed):
    """Steps of (request, tokens): every request's tokens in portions of the given sizes in turn, single tokens first in a step."""
    g = torch.Generator().manual_seed(seed)
    done, steps, i = [0] * len(lengths), [], 0
    while any(d < n for d, n in zip(done, lengths)):
        step = []
        for s, n in enumerate(lengths):
            if done[s] < n and (len(step) == 0 or torch.rand((), generator=g) < 0.8):
                q = min(portions[i % len(portions)], n - done[s])
                i += 1
                step.append((s, done[s], q))
                done[s] += q
        steps.append(sorted(step, key=lambda e: (e[2] != 1, e[0])))
    return steps


LIGHTNING_SIZES = [(3, 12, 10), (2, 128, 128), (3, 48, 160), (1, 64, 64), (4, 1, 24), (2, 100, 33), (2, 150, 20), (5, 17, 5)]


@BOTH
@pytest.mark.parametrize("H,d,dv", LIGHTNING_SIZES)
def test_lightning_recurrence(H, d, dv, dtype):
    """Requests of unequal length cut into portions, the walk and the chunks, rows of the state array in no order and used
    again, with the norm over all heads and the gate behind it.  Decays of 0 (nothing is kept), of 1 (everything is) and between."""
    from inferrs_amd import ops
    g = torch.Generator().manual_seed(H * d + dv)
    lengths = [1, 2, 17, 200, 333]
    decay = torch.tensor([1.0, 0.0, 0.999, 0.6, 3e-4][:H])
    qk, vv = H * d, H * dv
    ld = 2 * qk + 2 * vv + 8
    w = 1 + 0.3 * torch.randn(vv, generator=g)
    rows, want, states = [], [], []
    for n in lengths:
        r = torch.randn(n, ld, generator=g).to(dtype)
        r64 = r.double()
        q, k = (pl.silu(r64[:, i * qk:(i + 1) * qk]).view(n, H, d) for i in range(2))
        v = pl.silu(r64[:, 2 * qk:2 * qk + vv]).view(n, H, dv)
        o, S = pl.fading_sums(q, k, v, decay.double().tolist())
        rows.append(r); states.append(S)
        want.append(pl.rms_norm(o.reshape(n, vv), w.double(), 1e-5) * torch.sigmoid(r64[:, 2 * qk + vv:2 * qk + 2 * vv]))
    # (32-bit: a sum that nearly cancels keeps the rounding of its terms, and the norm divides a token's outputs by their size)
    rel = 1e-2 if dtype == torch.bfloat16 else 5e-5
    state = dev(torch.full((8, 4 + vv * d), 7.0))
    for portions, chunk in (([1000], None), ([1], 0), ([7, 1, 2, 40, 3, 1], 0), ([1000], 64), ([7, 1, 2, 150, 64, 3], 64), ([65, 1, 64, 63], 64), ([1000], 32)):
        slots_of = torch.randperm(7, generator=g)[:5].tolist()
        state[slots_of] = 0.0
        before = state.clone()
        for step in cut_steps(lengths, portions, seed=d):
            proj = dev(torch.cat([rows[s][a:a + q] for s, a, q in step]))
            o = ops.linear_scan(q=proj, q_off=0, q_heads=H, k=proj, k_off=qk, k_heads=H, v=proj, v_off=2 * qk, heads=H, dim=d, vdim=dv, state=state,
                                s_off=4, cu_tokens=i32(*np.cumsum([0] + [e[2] for e in step]).tolist()), state_slots=i32(*[slots_of[e[0]] for e in step]),
                                decay=dev(decay), max_q_len=max(e[2] for e in step), chunk=chunk, act=ops.state.ACT_SILU)
            got = ops.group_norm_gate(o, group=vv, head=dv, eps=1e-5, out_dtype=dtype, weight=dev(w), gate=proj, gate_off=2 * qk + vv,
                                      act=ops.state.ACT_SIGMOID)
            assert_close(got, torch.cat([want[s][a:a + q] for s, a, q in step]), rel, f"portions {portions}, chunk {chunk}")
        after = state.cpu()
        for s in range(len(lengths)):
            S = after[slots_of[s], 4:].view(H, dv, d).transpose(1, 2)
            assert_close(S, states[s], 2e-5, f"the state of request {s}, portions {portions}, chunk {chunk}")
        others = [i for i in range(8) if i not in slots_of]
        assert torch.equal(after[others], before.cpu()[others]) and bool((after[:, :4] == before.cpu()[:, :4]).all())


def test_lightning_reads_one_key_hundreds_of_tokens_later():
    """A value written once, in the walk and in the chunks: it fades by the head's constant a token, across every chunk's border."""
    from inferrs_amd import ops
    H, d, dv, n = 2, 32, 32, 450
    decay = torch.tensor([0.99, 1.0])
    for at in (0, 15, 16, 63, 64, 127, 200):
        rows = torch.zeros(n, 2 * H * d + H * dv)
        rows[:, 0] = rows[:, d] = 5.0                            # (each head's query looks along its first feature)
        rows[at, H * d] = rows[at, H * d + d] = 4.0              # one key, and its value
        rows[at, 2 * H * d:] = torch.linspace(1.0, 3.0, H * dv)
        q0, k0 = float(pl.silu(torch.tensor(5.0).double())), float(pl.silu(torch.tensor(4.0).double()))
        v0 = pl.silu(torch.linspace(1.0, 3.0, H * dv).double()).view(H, dv)
        for chunk in (0, 64):
            state = dev(torch.zeros(1, H * d * dv))
            x = dev(rows)
            got = ops.linear_scan(q=x, q_off=0, q_heads=H, k=x, k_off=H * d, k_heads=H, v=x, v_off=2 * H * d, heads=H, dim=d, vdim=dv, state=state,
                                  s_off=0, cu_tokens=i32(0, n), state_slots=i32(0), decay=dev(decay), max_q_len=n, chunk=chunk,
                                  act=ops.state.ACT_SILU).cpu().double().view(n, H, dv)
            assert bool((got[:at] == 0).all())
            for t in range(at, n):
                want = q0 * k0 * v0 * (decay.double() ** (t - at))[:, None]
                assert torch.allclose(got[t], want, rtol=2e-5 + 2e-7 * (t - at)), (at, t, chunk)


# ---- the router ---------------------------------------------------------------------------------------------------

GROUPS = [(6, 2, (3, 2), 48), (12, 5, (4, 2), 64), (64, 6, (8, 3), 136), (9, 4, (3, 3), 50), (6, 3, (2, 1), 50), (8, 2, (8, 3), 272), (4, 4, (1, 1), 40),
          (160, 8, (8, 4), 128), (200, 3, (100, 5), 48), (2, 1, (2, 1), 256)]


@BOTH
@pytest.mark.parametrize("E,top,groups,W", GROUPS)
def test_the_choice_inside_the_best_groups(E, top, groups, W, dtype):
    from inferrs_amd import ops
    g = torch.Generator().manual_seed(E * W)
    for n in (1, 9, 57, 200):
        h = torch.randn(n, W, generator=g).to(dtype)
        router = (2.5 * torch.randn(E, W, generator=g) / W ** 0.5).to(dtype)
        plan = ops.mix.ExpertPlan(n, top, E, True, torch.device("cuda"))
        sel, weight = ops.route(dev(h), dev(router), top, 1.7, "sigmoid", True, None, plan=plan, groups=groups)
        cfg = {"top": top, "scale": 1.7, "groups": {"count": groups[0], "keep": groups[1]}}
        chosen, want = pl.route(h.double(), {"router": router.double()}, "", cfg)
        s = torch.sigmoid(h.double() @ router.double().T)
        # rows without a close call: between groups, and between scores around the last one that is chosen
        size = E // groups[0]
        worth = torch.sort(s.view(n, groups[0], size), dim=-1, descending=True).values[:, :, :2].sum(-1)
        worth = torch.sort(worth, dim=-1, descending=True).values
        allowed = torch.sort(s.masked_fill(~pl.best_groups(s, *groups), -1.0), dim=-1, descending=True).values
        gaps = [allowed[:, :top] - torch.cat([allowed, torch.full((n, 1), -1.0)], 1)[:, 1:top + 1].to(s)]
        if groups[1] < groups[0]:
            gaps.append(worth[:, groups[1] - 1:groups[1]] - worth[:, groups[1]:groups[1] + 1])
        clear = torch.cat(gaps, dim=1).min(dim=1).values > 1e-5
        assert clear.float().mean() > 0.75 or n == 1
        assert torch.equal(sel.cpu().long()[clear], chosen[clear])
        np.testing.assert_allclose(weight.cpu()[clear].numpy(), want[clear].numpy(), rtol=2e-5, atol=1e-6)
        np.testing.assert_allclose(weight.cpu().sum(1).numpy(), 1.7, rtol=1e-5)
        # a choice from logits that another product has left makes the same of them
        if n <= ops.mix.ROUTE_LOGITS_ROWS:
            logits = dev(torch.cat([torch.zeros(n, 3), (h.double() @ router.double().T).float()], dim=1))
            sel2, weight2, _ = ops.mix.route_logits(logits, 3, E, top, 1.7, "sigmoid", True, None, 0,
                                                    ops.mix.ExpertPlan(n, top, E, True, torch.device("cuda")), groups=groups)
            assert torch.equal(sel2.cpu().long()[clear], chosen[clear])
            np.testing.assert_allclose(weight2.cpu()[clear].numpy(), want[clear].numpy(), rtol=2e-5, atol=1e-6)


def test_groups_with_a_correction_choose_by_corrected_scores_and_weigh_by_plain_ones():
    from inferrs_amd import ops
    g = torch.Generator().manual_seed(4)
    n, E, W, top, (count, keep) = 60, 16, 64, 3, (4, 2)
    h, router, bias = torch.randn(n, W, generator=g), 2 * torch.randn(E, W, generator=g) / 8, 0.3 * torch.randn(E, generator=g)
    sel, weight = ops.route(dev(h), dev(router), top, 1.0, "sigmoid", True, dev(bias), groups=(count, keep))
    s = torch.sigmoid(h.double() @ router.double().T)
    key = (s + bias.double()).masked_fill(~pl.best_groups(s + bias.double(), count, keep), float("-inf"))
    chosen = torch.topk(key, top, dim=-1).indices
    same = (sel.cpu().long() == chosen).all(1)
    assert same.float().mean() > 0.95
    won = torch.gather(s, 1, chosen)
    np.testing.assert_allclose(weight.cpu()[same].numpy(), (won / won.sum(-1, keepdim=True))[same].numpy(), rtol=2e-5)


def test_groups_that_do_not_fit_are_refused():
    from inferrs_amd import ops
    h, r = dev(torch.zeros(2, 16)), dev(torch.zeros(6, 16))
    for top, groups in ((2, (4, 2)), (3, (3, 1)), (1, (3, 4)), (1, (3, 0))):
        with pytest.raises(ops.KernelError, match="groups"):
            ops.route(h, r, top, 1.0, "sigmoid", True, groups=groups)


# ---- whole models under every cutting ---------------------------------------------------------------

_ROUNDED = {}
NOISE = {}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    out = {}
    for name, sharpen in CASES:
        cfg = sharpened(CONFIGS[name], sharpen)
        folder = str(tmp_path_factory.mktemp(f"lumedra_{name}"))
        tensors = write_model(folder, cfg, seed=11)
        reqs = {f"r{i}": random_tokens(n, cfg["vocab"], 40 + i) for i, n in enumerate(LENGTHS)}
        ref64 = {r: pl.forward(cfg, tensors, t) for r, t in reqs.items()}
        ref = {r: v.numpy().astype(np.float32) for r, v in ref64.items()}
        scale = max(float(v.abs().max()) for v in ref64.values())
        # what rounding alone does at every position: the plain implementation in 32-bit against itself in 64-bit
        # (the largest so far at every position: what a request carries is rounded on and on, and one position's error is one draw)
        NOISE[(name, sharpen)] = {r: np.maximum.accumulate(((pl.forward(cfg, tensors, t, dtype=torch.float32).double() - ref64[r])
                                                            .abs().max(1).values / scale).numpy()) for r, t in reqs.items()}
        out[(name, sharpen)] = (folder, cfg, tensors, reqs, ref)
    return out


def errors(got, ref, reqs):
    scale = max(float(np.abs(v).max()) for v in ref.values())
    return {r: np.array([float(np.abs(got[r][p] - ref[r][p]).max()) / scale for p in range(len(t))]) for r, t in reqs.items()}


def rounded_errors(key, models):
    """request -> the errors of the plain implementation in bfloat16 arithmetic, position by position."""
    if key not in _ROUNDED:
        folder, cfg, tensors, reqs, ref = models[key]
        some = {r: t for r, t in reqs.items() if len(t) <= 300}
        rounded = {r: pl.forward(cfg, tensors, t, dtype=torch.bfloat16).float().numpy() for r, t in some.items()}
        _ROUNDED[key] = errors(rounded, ref, some)
    return _ROUNDED[key]


def replay(folder, cfg, dtype, trace, out_dir, page=16, **kw):
    from inferrs_amd.engine import Engine, run_trace
    eng = Engine.from_folder(folder, dtype=dtype, page_size=page, num_pages=-(-trace.max_tokens // page), max_seqs=4, **kw)
    run_trace(eng, trace.lines, out_dir, io.StringIO())
    eng.cache.check_invariants()
    assert not eng.cache.sequences and all(g.pool.num_free == g.pool.num_pages for g in eng.cache.groups)
    assert eng.cache.slots.num_free == eng.cache.slots.num_slots
    return trace.read(out_dir, cfg["vocab"])


def traces(reqs):
    short = {r: t for r, t in reqs.items() if len(t) <= 65}
    return {
        "whole": tm.whole(reqs),
        "tail32": tm.prefix_then_single(reqs, 32),
        "every token alone": tm.prefix_then_single(short, 10 ** 6),
        "a long tail": tm.prefix_then_single({r: t for r, t in reqs.items() if 130 <= len(t) <= 300}, 120),
        "portions": tm.portions(reqs, [7, 2, 16, 3, 2, 33, 5, 2, 64]),
        "long portions": tm.portions({r: t for r, t in reqs.items() if len(t) >= 130}, [150, 2, 129]),
        "portions of two and three": tm.portions(short, [2, 3]),
        "mixed": tm.mixed(reqs, seed=1),
        "mixed2": tm.mixed(dict(reversed(list(reqs.items()))), seed=2, max_live=3),
    }


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("case", CASES, ids=lambda c: f"{c[0]}x{c[1]:g}")
def test_every_cutting_matches_plain(models, tmp_path, case, dtype):
    folder, cfg, tensors, reqs, ref = models[case]
    for mode, trace in traces(reqs).items():
        if mode.startswith("mixed"):
            assert trace.max_live >= 3 and trace.max_tokens < sum(tm.round_up(len(t), 64) for t in reqs.values())
        got = replay(folder, cfg, dtype, trace, str(tmp_path / f"{mode}_{dtype}"), page=16 if mode != "mixed2" else 32)
        part = {r: reqs[r] for r in got}
        if dtype == "float32":
            for r, e in errors(got, ref, part).items():
                allowed = np.maximum(TOL_F32, 3.0 * NOISE[case][r])
                assert (e <= allowed).all(), (f"{case} {dtype} {mode}: {float(e[np.argmax(e / allowed)]):.3g} of the scale at "
                                              f"({r}, {int(np.argmax(e / allowed))}), allowed {float(allowed[np.argmax(e / allowed)]):.3g}")
            continue
        plain = rounded_errors(case, models)
        common = [r for r in part if r in plain]
        mine = np.concatenate([errors(got, ref, part)[r] for r in common])
        theirs = np.concatenate([plain[r] for r in common])
        assert np.isfinite(np.concatenate(list(errors(got, ref, part).values()))).all(), f"{case} {mode}: not finite"
        for q, slack in ((0.5, 1.1), (0.9, 1.5)):
            a, b = float(np.quantile(mine, q)), float(np.quantile(theirs, q))
            assert a <= slack * b + 1e-3, f"{case} {dtype} {mode}: quantile {q} of the errors {a:.3g}, plain in bfloat16 {b:.3g}"


@pytest.mark.parametrize("case", [("A", 4.0), ("D", 2.5)], ids=lambda c: f"{c[0]}x{c[1]:g}")
def test_the_models_rest_on_what_the_tests_are_for(models, case):
    """A first key that is lost, a window one token off, values that are not mixed, a decay one step off, a group too many, a
    norm taken for the other: each moves the logits by far more than any tolerance above."""
    folder, cfg, tensors, reqs, ref = models[case]
    toks = reqs["r7"]
    scale = float(np.abs(ref["r7"]).max())
    allowed = 100 * max(TOL_F32, float(NOISE[case]["r7"].max()))

    def moved(other_cfg=None, **other):
        w = dict(tensors, **{k.replace("__", "."): v for k, v in other.items()})
        return float(np.abs(pl.forward(other_cfg or cfg, w, toks).numpy() - ref["r7"]).max()) / scale

    def changed(kind, change):
        c = json.loads(json.dumps(cfg))
        for L in c["layers"]:
            if L["type"] == kind:
                change(L["mixer"])
                break
        return c

    assert moved(changed("attention", lambda m: m["mask"].__setitem__("keep_first", m["mask"]["keep_first"] - 1))) > allowed
    assert moved(changed("attention", lambda m: m["mask"].__setitem__("size", m["mask"]["size"] + 1))) > allowed
    assert moved(changed("attention", lambda m: m.__setitem__("softcap", 1.2 * m["softcap"]))) > allowed
    assert moved(changed("attention", lambda m: m.__setitem__("v_mix", False))) > allowed
    assert moved(changed("lightning", lambda m: m.__setitem__("decay", [0.99 * d for d in m["decay"]]))) > allowed
    c = json.loads(json.dumps(cfg))
    for L in c["layers"]:
        if L["mlp"] and L["mlp"]["kind"] == "moe":
            L["mlp"]["router"].pop("groups", None)
    assert moved(c) > allowed
    assert moved(l0__norm2=tensors["l0.norm1"]) > allowed


@pytest.mark.parametrize("name", ["A", "C", "D"])
def test_greedy_generation_through_the_scheduler(models, name):
    from inferrs_amd.engine import Engine
    from inferrs_amd.sampling import SamplingParams
    folder, cfg, tensors, reqs, ref = models[(name, 1.0)]
    prompts = [random_tokens(n, cfg["vocab"], 900 + n) for n in (1, 5, 40, 90, 17, 64)]
    n_new = [12, 30, 7, 20, 25, 3]
    eng = Engine.from_folder(folder, dtype="float32", page_size=8, num_pages=40, max_seqs=4)
    outs = eng.generate(prompts, [SamplingParams.greedy(max_tokens=n, bypass_stop_tokens=True) for n in n_new],
                        max_batch_size=3, max_tokens_per_step=48, prefill_chunk=16)
    for prompt, n, out in zip(prompts, n_new, outs):
        toks = list(prompt)
        for _ in range(n):
            toks.append(int(pl.forward(cfg, tensors, toks)[-1].argmax()))
        assert out.error is None and out.tokens == toks[len(prompt):]
    eng.cache.check_invariants()
    assert not eng.cache.sequences and eng.cache.slots.num_free == eng.cache.slots.num_slots


def test_decode_steps_replayed_from_graphs(models):
    """Generation with the serving loop's graphs against the same engine without them.  32-bit: the same sums in the
    same order, so the same tokens.  bfloat16: a graph's step sees its context bucket's width and an eager step the
    longest request, so keys may be split between waves in another way; given tokens are fed and the logits compared."""
    from inferrs_amd.engine import Engine
    from inferrs_amd.engine.engine import Entry
    from inferrs_amd.sampling import SamplingParams
    folder, cfg, tensors, reqs, ref = models[("D", 1.0)]
    prompts = [random_tokens(n, cfg["vocab"], 700 + n) for n in (33, 5, 120)]
    outs = []
    for graphs in (False, True):
        eng = Engine.from_folder(folder, dtype="float32", page_size=16, num_pages=64, max_seqs=4, use_graphs=graphs)
        assert eng.use_graphs == graphs
        res = eng.generate(prompts, [SamplingParams.greedy(max_tokens=40, bypass_stop_tokens=True)] * 3, max_batch_size=3)
        assert all(o.error is None for o in res) and (eng.graph_replays > 20) == graphs
        outs.append([o.tokens for o in res])
    assert outs[0] == outs[1]
    toks = reqs["r7"]                                    # 300 tokens: 250 as a prompt, 50 fed one by one
    want = ref["r7"][249:]
    scale = float(np.abs(ref["r7"]).max())
    for graphs in (False, True):
        eng = Engine.from_folder(folder, dtype="bfloat16", page_size=16, num_pages=64, max_seqs=4, use_graphs=graphs)
        rows = [eng.step([Entry("a", toks[:250], [249])])[0].clone()]
        rows += [eng.step([Entry("a", [t], [0])])[0].clone() for t in toks[250:]]
        assert (eng.graph_replays > 20) == graphs
        err = np.abs(torch.stack(rows).cpu().numpy() - want).max(1) / scale
        assert float(np.median(err)) <= 5e-2, (graphs, float(np.median(err)))


def test_random_weights_engine_steps():
    """The measurement script's way in: a configuration object and weights drawn on the device."""
    from inferrs_amd.config.lumedra import LumedraConfig
    from inferrs_amd.engine import Engine
    from inferrs_amd.engine.engine import Entry
    eng = Engine.from_random(LumedraConfig.from_dict(CONFIGS["A"]), seed=1, dtype="bfloat16", page_size=16, num_pages=16, max_seqs=2)
    logits = eng.step([Entry("a", random_tokens(33, 199, 1), [32]), Entry("b", [5], [0])])
    assert logits.shape == (2, 199) and bool(torch.isfinite(logits).all())


def test_command_line_run_and_bench(models):
    """The command line serves the design as it serves the others: greedy tokens are the plain implementation's, a drawn run
    and the timing command finish."""
    folder, cfg, tensors, reqs, ref = models[("A", 1.0)]
    prompt = random_tokens(9, cfg["vocab"], 3)
    toks = list(prompt)
    for _ in range(6):
        toks.append(int(pl.forward(cfg, tensors, toks)[-1].argmax()))
    exe = [sys.executable, os.path.join(ROOT, "bin", "inferrs-amd")]
    common = ["--block-size", "16", "--max-blocks", "32", "--max-batch-size", "2"]
    proc = subprocess.run(exe + ["run", folder, ",".join(map(str, prompt)), "--dtype", "f32", "--temperature", "0",
                                 "--repetition-penalty", "1.0", "--max-tokens", "6"] + common, capture_output=True, text=True, timeout=300)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [int(t) for t in proc.stdout.split()] == toks[len(prompt):]
    proc = subprocess.run(exe + ["run", folder, ",".join(map(str, prompt)), "--dtype", "bf16", "--seed", "5", "--max-tokens", "12",
                                 "--ignore-eos"] + common, capture_output=True, text=True, timeout=300)
    assert proc.returncode == 0, proc.stderr[-2000:]
    drawn = [int(t) for t in proc.stdout.split()]
    assert len(drawn) == 12 and all(0 <= t < cfg["vocab"] for t in drawn)
    proc = subprocess.run(exe + ["bench", folder, "--dtype", "bf16", "--prompt-len", "40", "--max-tokens", "8", "--runs", "2"] + common,
                          capture_output=True, text=True, timeout=300)
    assert proc.returncode == 0, proc.stderr[-2000:]
    rec = json.loads(proc.stdout.strip().splitlines()[-1])
    assert rec["prefill_tok_s"] > 0 and rec["decode_tok_s"] > 0


def test_trace_runner_program(models, tmp_path):
    folder, cfg, tensors, reqs, ref = models[("C", 1.0)]
    some = {r: reqs[r] for r in ("r2", "r3", "r4")}
    trace = tm.mixed(some, seed=5, max_live=2)
    out_dir = str(tmp_path / "out")
    p = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", "float32", "--out", out_dir,
                        "--max-tokens", str(trace.max_tokens)], input=trace.text(), capture_output=True, text=True, timeout=600)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(len(trace.lines))]
    for r, e in errors(trace.read(out_dir, cfg["vocab"]), ref, some).items():
        assert (e <= np.maximum(TOL_F32, 3.0 * NOISE[("C", 1.0)][r])).all(), (r, float(e.max()))
