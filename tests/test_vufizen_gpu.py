"""Vufizen on the GPU against the plain implementation (`plain_vufizen.py`, 64-bit).

Mechanisms alone, through the kernels' Python face: the kernel that closes a sub-layer (every addend, products still split
along their k, routed rows, a gated second output, with and without a gate), what stands between the projections and the
attention (the convolution over a request's cut portions, the norm a map, the turn, queries that are zero outside their map,
keys and values in shuffled pages), the combination of two maps, differential attention as a whole with keys that stand out
far away, at page borders and in one map only, the recurrence in its walk and in its chunks (portions cut anywhere, gates
that close, open or do neither, several passes over the chunks, slots used again), the router's softmax over the chosen
logits, the experts without limits.  Then whole models through the engine's step function under every way of cutting the
work (whole prompts, a prompt and then token by token, every token alone, portions down to two tokens, up to four live
requests mixed in a pool whose pages and slots are used again), in both precisions, with ordinary weights and with sharpened
queries.  Greedy generation runs through the engine's own entry point and scheduler, the command line and the replay program.

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

import plain_vufizen as pv
import trace_modes as tm
from vufizen_configs import CONFIGS, random_tokens, sharpened, write_model

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
LENGTHS = [1, 2, 3, 17, 64, 65, 130, 300, 700]
TOL_F32 = 2e-5
CASES = [("A", 1.0), ("B", 1.0), ("C", 1.0), ("D", 1.0), ("E", 1.0), ("A", 4.0), ("D", 2.5)]
BOTH = pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])


def dev(t, dtype=None):
    return t.to(device="cuda", dtype=dtype or t.dtype).contiguous()


def i32(*v):
    return dev(torch.tensor(v, dtype=torch.int32))


def assert_close(got, want, rel, what):
    err = float((got.double().cpu() - want).abs().max()) / max(float(want.abs().max()), 1e-9)
    assert err <= rel, f"{what}: {err:.3g} of the scale, allowed {rel:.3g}"


# ---- the kernel that closes a sub-layer --------------------------------------------------------------------

@pytest.mark.parametrize("W", [40, 33, 304, 5000, 9000])
@BOTH
def test_branch_step(W, dtype):
    from inferrs_amd import ops
    g = torch.Generator().manual_seed(W)
    n, top = 13, 3
    x = 3 * torch.randn(n, W, generator=g) + 0.7
    y, y3 = (torch.randn(n, W, generator=g).to(dtype) for _ in range(2))
    rows = (2 * torch.randn(n, W + 16, generator=g)).to(dtype)            # (the gate lies in rows of its mixer's product)
    routed, rw, s3 = torch.randn(n, top, W, generator=g), torch.rand(n, top, generator=g), torch.rand(n, generator=g)
    b, w = torch.randn(W, generator=g), 0.5 + torch.rand(W, generator=g)
    gate = torch.sigmoid(rows.double()[:, 16:] + b.double())

    def closed(s, gated=True):
        return x.double() + pv.rms_norm(s * gate if gated else s, w.double(), 1e-5)

    def run(**adds):
        xs = dev(x)
        xr = ops.branch_step(xs, weight=dev(w), eps=1e-5, **adds)
        return xs, xr

    gates = dict(gate=dev(rows), gate_off=16, gate_bias=dev(b))
    xs, xr = run(y=dev(y), x_dtype=dtype, **gates)
    assert_close(xs, closed(y.double()), 2e-6, "a dense output behind its gate")
    assert_close(xr, closed(y.double()), 5e-3 if dtype == torch.bfloat16 else 2e-6, "the rows once more")
    xs, xr = run(y=dev(y))
    assert xr is None
    assert_close(xs, closed(y.double(), False), 2e-6, "no gate")
    want = (rw.double()[:, :, None] * routed.double()).sum(1)
    xs, _ = run(routed=dev(routed), routed_weights=dev(rw), **gates)
    assert_close(xs, closed(want), 2e-6, "routed rows")
    xs, xr = run(routed=dev(routed), routed_weights=dev(rw), y3=dev(y3), y3_scale=dev(s3), x_dtype=dtype, **gates)
    assert_close(xs, closed(want + s3.double()[:, None] * y3.double()), 2e-6, "routed rows and a gated output beside them")
    parts, parts3 = torch.randn(3, n, W, generator=g), torch.randn(2, n, W, generator=g)
    xs, _ = run(y=ops.Partials(dev(parts)), x_dtype=dtype, **gates)
    assert_close(xs, closed(parts.double().sum(0)), 2e-6, "a product still split along its k")
    xs, _ = run(routed=dev(routed), routed_weights=dev(rw), y3=ops.Partials(dev(parts3)), y3_scale=dev(s3), x_dtype=dtype, **gates)
    assert_close(xs, closed(want + s3.double()[:, None] * parts3.double().sum(0)), 2e-6, "routed rows and a split output")
    # a row of zeros stays: the norm's eps keeps its root away from zero
    xs, _ = run(y=dev(torch.zeros(n, W, dtype=dtype)), **gates)
    assert torch.equal(xs.cpu(), x)


# ---- between the projections and the attention -------------------------------------------------------------

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


CONV_SIZES = [(4, 2, 8, 12, 4, 6, True), (3, 3, 11, 13, 3, 10, True), (4, 1, 64, 128, 4, 32, True), (4, 2, 24, 48, 6, 0, True),
              (2, 1, 16, 8, 1, 16, True), (4, 4, 16, 24, 2, 16, False), (1, 1, 128, 256, 4, 128, True), (2, 2, 6, 9, 5, 4, False)]


@BOTH
@pytest.mark.parametrize("H,G,d,dv,k,turned,neighbours", CONV_SIZES)
def test_convolution_norm_turn_and_cache(H, G, d, dv, k, turned, neighbours, dtype):
    from inferrs_amd import ops
    g = torch.Generator().manual_seed(H * d + k)
    C, ld, page, eps = 2 * (H + G) * d + G * dv, 2 * (H + G) * d + G * dv + 24, 8, 1e-5
    lengths = [37, 1, 2, 60, 5]
    rows = [torch.randn(n, ld, generator=g).to(dtype) for n in lengths]
    taps = (torch.randn(C, k, generator=g) / k ** 0.5).to(dtype)
    qn, kn = 1 + 0.3 * torch.randn(d, generator=g), 1 + 0.3 * torch.randn(d, generator=g)
    rot = {"base": 777.0, "dims": turned} if turned else None
    want_q, want_k, want_v = [], [], []
    for r in rows:
        n = r.shape[0]
        u = pv.short_convolution(r.double()[:, :C], taps.double())
        pos = torch.arange(n)
        q = pv.rms_norm(u[:, :2 * H * d].view(n, H, 2, d), qn.double(), eps)
        kk = pv.rms_norm(u[:, 2 * H * d:2 * (H + G) * d].view(n, G, 2, d), kn.double(), eps)
        if turned and neighbours:
            q, kk = pv.turn(q, pos, rot), pv.turn(kk, pos, rot)
        elif turned:                              # (halves paired: the same turn on reordered features)
            order = torch.cat([torch.arange(turned).view(2, -1).t().flatten(), torch.arange(turned, d)])
            back = torch.argsort(order)
            q, kk = (pv.turn(t[..., order], pos, rot)[..., back] for t in (q, kk))
        wide = torch.zeros(n, H, 2, 2, d, dtype=torch.float64)
        wide[:, :, 0, 0], wide[:, :, 1, 1] = q[:, :, 0], q[:, :, 1]
        want_q.append(wide.view(n, 2 * H, 2 * d)); want_k.append(kk.reshape(n, G, 2 * d)); want_v.append(u[:, 2 * (H + G) * d:].view(n, G, dv))
    rel = 1e-2 if dtype == torch.bfloat16 else 5e-6
    for portions in ([1000], [1], [7, 1, 2, 16, 3, 1]):
        slots_of, pages = [2, 0, 5, 3, 1], 40                     # (state rows and pages in no order)
        perm = torch.randperm(pages * page // 8, generator=g).tolist()
        table = {s: [perm.pop() for _ in range(-(-n // page))] for s, n in enumerate(lengths)}
        row_floats = -(-(k - 1) * C // 4) * 4 + 4
        state = dev(torch.zeros(6, row_floats)) if k > 1 else None
        kc, vc = dev(torch.zeros(pages, G, page, 2 * d, dtype=dtype)), dev(torch.zeros(pages, G, dv, page, dtype=dtype))
        for step in cut_steps(lengths, portions, seed=k):
            proj = torch.cat([rows[s][a:a + q] for s, a, q in step])
            pos = torch.cat([torch.arange(a, a + q) for s, a, q in step])
            slots = torch.tensor([table[s][p // page] * page + p % page for s, a, q in step for p in range(a, a + q)], dtype=torch.int32)
            cos = sin = None
            if turned:
                ang = pos.double()[:, None] * torch.tensor([777.0 ** (-2.0 * i / turned) for i in range(turned // 2)])[None, :]
                cos, sin = dev(torch.cos(ang).float()), dev(torch.sin(ang).float())
            q_out = ops.conv_qkv(dev(proj), dev(taps.t().contiguous()), state, 4 if k > 1 else 0, heads=H, kv_heads=G, maps=2, dim=d, vdim=dv,
                                 q_norm_w=dev(qn), k_norm_w=dev(kn), eps=eps, cos=cos, sin=sin, rot=turned, interleaved=neighbours,
                                 k_cache=kc, v_cache=vc, slots=dev(slots), page_size=page,
                                 token_seq=i32(*[j for j, e in enumerate(step) for _ in range(e[2])]),
                                 cu_tokens=i32(*np.cumsum([0] + [e[2] for e in step]).tolist()), state_slots=i32(*[slots_of[e[0]] for e in step]),
                                 max_q_len=max(e[2] for e in step))
            want = torch.cat([want_q[s][a:a + q] for s, a, q in step])
            assert_close(q_out, want, rel, f"queries, portions {portions}")
            assert bool((q_out.cpu()[want == 0] == 0).all())             # exactly zero outside the map
        for s, n in enumerate(lengths):
            at = torch.tensor([table[s][p // page] for p in range(n)]), torch.arange(n) % page
            assert_close(kc.cpu()[at[0], :, at[1]], want_k[s], rel, f"keys, portions {portions}")
            assert_close(vc.cpu()[at[0], :, :, at[1]], want_v[s], rel, f"values, portions {portions}")
            if k > 1:                             # what the request keeps: its last inputs as they came, zeros before the start
                kept = torch.cat([torch.zeros(max(k - 1 - n, 0), C), rows[s][max(n - k + 1, 0):, :C].float()])
                assert torch.equal(state.cpu()[slots_of[s], 4:4 + (k - 1) * C].view(k - 1, C), kept)
        if k > 1:
            assert bool((state.cpu()[4] == 0).all()) and bool((state.cpu()[:, :4] == 0).all())   # (a row of nobody's, and what lies before)


@BOTH
@pytest.mark.parametrize("H,dv", [(4, 12), (3, 13), (2, 128), (5, 64), (1, 256), (2, 264)])
def test_second_map_off_the_first(H, dv, dtype):
    from inferrs_amd import ops
    g = torch.Generator().manual_seed(dv)
    a = torch.randn(21, 2 * H, dv, generator=g).to(dtype)
    a[3, 0] = a[3, 1]                                               # (equal maps with lambda 1 leave zeros)
    for lam, diff in ((0.37, 0.5), (1.0, 0.2), (-0.4, 0.0)):
        got = ops.differ_norm(dev(a), lam, 1e-5, 1.0 - diff)
        pairs = a.double().view(21, H, 2, dv)
        want = pv.differ(pairs[:, :, 0], pairs[:, :, 1], lam, diff, 1e-5)
        assert_close(got, want.reshape(21, H * dv), 5e-3 if dtype == torch.bfloat16 else 1e-5, f"lambda {lam}")


@BOTH
@pytest.mark.parametrize("H,G,d,dv,n", [(4, 2, 8, 12, 70), (4, 1, 64, 128, 700), (2, 2, 32, 64, 300), (3, 3, 11, 13, 90), (6, 2, 24, 48, 260)])
def test_differential_attention(H, G, d, dv, n, dtype):
    """The kernels together, from the projections' rows on (one tap, so that what is planted stays): a key of one map only that
    stands out, far away and at page borders, for single tokens and for portions, over shuffled pages whose unwritten slots
    hold NaN."""
    from inferrs_amd import ops
    from inferrs_amd.parts.attention import Attention
    from inferrs_amd.config.spec import AttentionSpec, PositionSpec
    g = torch.Generator().manual_seed(n + d)
    C, page, eps, lam, diff, scale = 2 * (H + G) * d + G * dv, 16, 1e-5, 0.45, 0.6, d ** -0.5 * 2
    rows = torch.randn(n, C, generator=g)
    ones = torch.ones(d)
    # head 0's query of map m at these positions looks for this key's map m alone (the norm keeps the direction)
    planted = [(n - 1, 0, 0), (n - 2, 15, 1), (n - 3, 16, 0), (n // 2, n // 2 - 17, 1), (n // 2 + 1, n // 2 + 1, 0)]
    qv = rows[:, :2 * H * d].view(n, H, 2, d)
    kv = rows[:, 2 * H * d:2 * (H + G) * d].view(n, G, 2, d)
    for i, j, m in planted:
        kv[j, 0, m] = qv[i, 0, m]
    rows = rows.to(dtype)
    # the plain implementation from h on: projections that pick the rows' parts
    eye = torch.eye(C, dtype=torch.float64)
    w = {"q": eye[:2 * H * d], "k": eye[2 * H * d:2 * (H + G) * d], "v": eye[2 * (H + G) * d:], "q.norm": ones.double(), "k.norm": ones.double(),
         "o": torch.eye(H * dv, dtype=torch.float64), "lq1": torch.zeros(d), "lk1": torch.zeros(d), "lq2": torch.zeros(d), "lk2": torch.zeros(d)}
    w.update({x + ".conv": torch.ones(w[x].shape[0], 1, dtype=torch.float64) for x in ("q", "k", "v")})
    w["lq1"][0], w["lk1"][0] = 1.0, float(np.log(lam - diff + 1.0))         # exp(lq1 . lk1) - exp(0) + diff = lam
    w = {k: v.double() for k, v in w.items()}
    m = {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "diff": diff, "scale": scale}
    want = pv.differential_attention(rows.double(), w, "", m, eps)
    for i, j, mm in planted:                                           # (each planted key is worth something where it is looked for)
        other = rows.double().clone()
        other[j, 2 * H * d + mm * d:2 * H * d + (mm + 1) * d] *= -1
        assert float((pv.differential_attention(other, w, "", m, eps) - want)[i].abs().max()) > 0.05, (i, j, mm)
    pages = -(-n // page)
    perm = torch.randperm(pages + 2, generator=g)[:pages]
    spec = AttentionSpec(hidden=8, n_heads=2 * H, n_kv_heads=G, head_dim=2 * d, position=PositionSpec("none"), scale=scale, v_head_dim=dv)
    rel = 4e-2 if dtype == torch.bfloat16 else 3e-5

    class Step:
        pass

    for portions in ([n], [n - 40] + [1] * 40, [33, 2, 100, 5, 64]):
        kc, vc = (dev(torch.full(s, float("nan"), dtype=dtype)) for s in ((pages + 2, G, page, 2 * d), (pages + 2, G, dv, page)))
        at, i = 0, 0
        while at < n:
            q_len = min(portions[i % len(portions)], n - at)
            i += 1
            pos = torch.arange(at, at + q_len, dtype=torch.int32)
            ctx, group = Step(), Step()
            ctx.positions, ctx.token_seq, ctx.cu_tokens = dev(pos), dev(torch.zeros(q_len, dtype=torch.int32)), i32(0, q_len)
            ctx.n_single, ctx.n_seqs, ctx.n_tokens, ctx.max_q_len, ctx.max_kv_len = int(q_len == 1), 1, q_len, q_len, at + q_len
            ctx.max_kv_single = ctx.max_kv_multi = at + q_len
            group.page_size, group.block_table = page, dev(perm.to(torch.int32)[None, :].contiguous())
            group.slots = dev((perm[pos.long() // page] * page + pos % page).to(torch.int32))
            q = ops.conv_qkv(dev(rows[at:at + q_len]), dev(torch.ones(1, C, dtype=dtype)), None, 0, heads=H, kv_heads=G, maps=2, dim=d, vdim=dv,
                             q_norm_w=dev(ones), k_norm_w=dev(ones), eps=eps, cos=None, sin=None, rot=0, interleaved=True, k_cache=kc,
                             v_cache=vc, slots=group.slots, page_size=page, token_seq=ctx.token_seq, cu_tokens=ctx.cu_tokens,
                             state_slots=i32(0), max_q_len=q_len)
            cache = Step()
            cache.k, cache.v = kc, vc
            got = ops.differ_norm(Attention.attend(spec, ctx, q, cache, group), lam, eps, 1.0 - diff)
            assert_close(got, want[at:at + q_len], rel, f"portions {portions[:3]} at {at}")
            at += q_len


# ---- the recurrence ---------------------------------------------------------------------------------------------

FADING_SIZES = [(3, 12, 10), (2, 128, 128), (2, 48, 160), (1, 64, 64), (4, 1, 24), (2, 100, 33), (2, 150, 20), (3, 17, 256), (2, 16, 5)]


@BOTH
@pytest.mark.parametrize("H,d,dv", FADING_SIZES)
def test_fading_recurrence(H, d, dv, dtype, monkeypatch):
    """Requests of unequal length cut into portions, the walk and the chunks, rows of the state array in no order and used again.
    Channels remember everything (gates within 1e-6 of one), nothing (floors of zero and closed gates), or fade at every rate
    in between within a head."""
    from inferrs_amd import ops
    g = torch.Generator().manual_seed(H * d + dv)
    lengths = [1, 2, 17, 200, 333]
    ld = 2 * H * d + H * dv + 8
    fb = 8.0 * torch.rand(H * d, generator=g) - 2.0
    lower = torch.rand(H * d, generator=g) ** 2
    fb[::5], lower[::5] = 14.0, 0.3
    fb[1::7], lower[1::7] = -40.0, 0.0
    lower[2::7] = 1.0                                    # (a channel whose gate cannot open: it holds its zeros)
    w = 1 + 0.3 * torch.randn(dv, generator=g)
    rows, want, states = [], [], []
    for n in lengths:
        r = torch.randn(n, ld, generator=g).to(dtype)
        if n > 20:
            r[n // 2, H * d:2 * H * d] = 60.0            # a token at which every channel holds
            r[n // 2 + 1, H * d:2 * H * d] = -60.0       # and one at which every channel lets go down to its floor
        r64 = r.double()
        q = pv.silu(r64[:, :H * d]).view(n, H, d)
        low = lower.double()
        f = (low + (1 - low) * torch.sigmoid(r64[:, H * d:2 * H * d] + fb.double())).view(n, H, d)
        o, S = pv.fading_outer_products(q, f, r64[:, 2 * H * d:2 * H * d + H * dv].view(n, H, dv))
        rows.append(r); want.append(pv.rms_norm(o, w.double(), 1e-5).reshape(n, H * dv)); states.append(S)
    fits = d <= 128 and dv <= 256
    rel = 1e-2 if dtype == torch.bfloat16 else 2e-5
    cases = [([1000], None), ([1], False), ([7, 1, 2, 40, 3, 1], False)]
    if fits:
        cases += [([1000], True), ([7, 1, 2, 150, 64, 3], True), ([65, 1, 64, 63], True), ([1000], "passes")]
    state = dev(torch.full((8, 8 + H * dv * d), 7.0))
    for portions, chunks in cases:
        if chunks == "passes":                           # (room for two chunks of every request at a time)
            monkeypatch.setattr(ops.gated, "FADING_WORKSPACE_FLOATS", 2 * len(lengths) * H * d * (dv + 1))
            chunks = True
        slots_of = torch.randperm(7, generator=g)[:5].tolist()
        state[slots_of] = 0.0
        before = state.clone()
        for step in cut_steps(lengths, portions, seed=d):
            got = ops.fading_scan(dev(torch.cat([rows[s][a:a + q] for s, a, q in step])), q_off=0, f_off=H * d, v_off=2 * H * d, heads=H, dim=d,
                                  vdim=dv, f_bias=dev(fb), lower=dev(lower), norm_weight=dev(w), eps=1e-5, state=state, s_off=4,
                                  cu_tokens=i32(*np.cumsum([0] + [e[2] for e in step]).tolist()), state_slots=i32(*[slots_of[e[0]] for e in step]),
                                  max_q_len=max(e[2] for e in step), chunks=chunks)
            assert got.dtype == dtype
            assert_close(got, torch.cat([want[s][a:a + q] for s, a, q in step]), rel, f"portions {portions}, chunks {chunks}")
        after = state.cpu()
        for s in range(len(lengths)):
            S = after[slots_of[s], 4:4 + H * dv * d].view(H, dv, d).transpose(1, 2)
            assert_close(S, states[s], 2e-5, f"the state of request {s}, portions {portions}, chunks {chunks}")
        others = [i for i in range(8) if i not in slots_of]
        assert torch.equal(after[others], before.cpu()[others])
        assert bool((after[:, :4] == before.cpu()[:, :4]).all()) and bool((after[:, 4 + H * dv * d:] == before.cpu()[:, 4 + H * dv * d:]).all())


def test_fading_recurrence_remembers_one_token():
    """A value written once, hundreds of tokens back, in the walk and in the chunks: channels whose gates stay shut behind it
    hold it exactly, and a chunk's or a block's border before or behind it loses nothing."""
    from inferrs_amd import ops
    H, d, dv, n = 1, 32, 32, 450
    fb, lower, w = torch.zeros(d), torch.zeros(d), torch.ones(dv)
    for at in (0, 15, 16, 63, 64, 127, 200):
        rows = torch.zeros(n, 2 * d + dv)
        rows[:, :d] = 5.0
        rows[:, d:2 * d] = 80.0                                # (gates held shut: f = 1)
        rows[at, d:2 * d] = 0.0                                # one token at which they are half open
        rows[at, 2 * d:] = torch.arange(1.0, dv + 1)
        for chunks in (False, True):
            state = dev(torch.zeros(1, d * dv))
            got = ops.fading_scan(dev(rows), q_off=0, f_off=d, v_off=2 * d, heads=H, dim=d, vdim=dv, f_bias=dev(fb), lower=dev(lower),
                                  norm_weight=dev(w), eps=1e-9, state=state, s_off=0, cu_tokens=i32(0, n), state_slots=i32(0),
                                  max_q_len=n, chunks=chunks).cpu()
            v = torch.arange(1.0, dv + 1)
            assert bool((got[:at] == 0).all())
            assert torch.allclose(got[at:], (v / (v * v).mean().sqrt()).expand(n - at, dv), rtol=1e-5), (at, chunks)
            assert torch.equal(state.cpu().view(dv, d), 0.5 * v[:, None].expand(dv, d))


# ---- the router and the experts ---------------------------------------------------------------------------------

@BOTH
@pytest.mark.parametrize("E,top,W", [(5, 2, 48), (1, 1, 64), (3, 3, 50), (70, 6, 136), (11, 3, 272)])
def test_router_softmax_over_the_chosen(E, top, W, dtype):
    from inferrs_amd import ops
    g = torch.Generator().manual_seed(E * W)
    for n in (1, 57, 200):
        h = torch.randn(n, W, generator=g).to(dtype)
        w = {"router": (3 * torch.randn(E, W, generator=g) / W ** 0.5).to(dtype).double()}
        gate = torch.randn(1, W, generator=g).to(dtype)
        sel, weight, sg = ops.route(dev(h), dev(torch.cat([w["router"].to(dtype), gate])), top, 1.0, "softmax", True, None, gates=1)
        chosen, want = pv.route(h.double(), w, "", top)
        z = torch.sort(h.double() @ w["router"].T, dim=-1, descending=True).values
        clear = ((z[:, :-1] - z[:, 1:])[:, :top].abs().min(dim=1).values > 1e-4) if E > 1 else torch.ones(n, dtype=torch.bool)
        assert clear.float().mean() > 0.8
        assert torch.equal(sel.cpu().long()[clear], chosen[clear])
        np.testing.assert_allclose(weight.cpu()[clear].numpy(), want[clear].numpy(), rtol=1e-4, atol=1e-6)
        np.testing.assert_allclose(weight.cpu().sum(1).numpy(), 1.0, rtol=1e-5)
        np.testing.assert_allclose(sg.cpu().numpy(), torch.sigmoid(h.double() @ gate.double().T).numpy(), rtol=1e-4, atol=1e-6)


@pytest.mark.parametrize("E,top,n", [(11, 5, 16), (33, 1, 5), (63, 8, 1), (2, 2, 9)])
def test_the_router_makes_the_plan_of_a_short_step(E, top, n):
    """The pairs ordered by expert and the table of row tiles, made on the way by the router's kernel: what the kernel of its
    own makes of the same choices (the pairs of an expert in any order)."""
    from inferrs_amd import ops
    g = torch.Generator().manual_seed(E)
    h, router = torch.randn(n, 256, generator=g).bfloat16(), torch.randn(E + 1, 256, generator=g).bfloat16()
    made = ops.mix.ExpertPlan(n, top, E, True, torch.device("cuda"))
    sel, weight, gate = ops.route(dev(h), dev(router), top, 1.0, "softmax", True, None, gates=1, plan=made)
    assert made.done
    own = ops.mix.ExpertPlan(n, top, E, True, torch.device("cuda"))
    order, expert, first, rows, meta = own.parts
    ops._check(ops.library().ia_route_plan(*(ops._p(t) for t in own.parts), ops._p(sel), n * top, E, own.tile, ops._stream()))
    tiles = int(meta[0])
    assert int(made.parts[4][0]) == tiles
    assert all(torch.equal(made.parts[i][:tiles], own.parts[i][:tiles]) for i in (1, 2, 3))
    flat = sel.flatten().cpu()
    for plan in (made, own):
        o = plan.parts[0].cpu().long()
        assert sorted(o.tolist()) == list(range(n * top)) and torch.equal(flat[o], torch.sort(flat).values)


@BOTH
@pytest.mark.parametrize("E,top,W,ff", [(5, 2, 48, 24), (3, 3, 50, 30), (6, 2, 64, 32), (10, 1, 384, 48)])
def test_experts_without_limits(E, top, W, ff, dtype):
    from inferrs_amd import ops
    g = torch.Generator().manual_seed(E + ff)
    for n in (1, 9, 150):
        h = (4 * torch.randn(n, W, generator=g)).to(dtype)
        sel = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(n)]).to(torch.int32)
        gu = (2 * torch.randn(E, 2 * ff, W, generator=g) / W ** 0.5).to(dtype)
        down = (torch.randn(E, W, ff, generator=g) / ff ** 0.5).to(dtype)
        tiled = ops.mix.experts_tiled_fits(dtype, W, ff)
        a, b = dev(gu), dev(down)
        if tiled:
            a, b = ops.mix.tile_weights(a.view(E, 2, ff, W)), ops.mix.tile_weights(b)
        y = ops.experts_forward(dev(h), dev(sel), a, b, 7.0, 1.702, ff=ff if tiled else None, activation="silu").cpu()
        for t in range(n):
            for k in range(top):
                e = int(sel[t, k])
                w = {"gate": gu[e, :ff].double(), "up": gu[e, ff:].double(), "down": down[e].double()}
                assert_close(y[t, k], pv.expert(h[t:t + 1].double(), w, "")[0], 2e-2 if dtype == torch.bfloat16 else 2e-5, f"n={n} ({t}, {k})")


# ---- whole models under every cutting ---------------------------------------------------------------

_ROUNDED = {}
NOISE = {}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    out = {}
    for name, sharpen in CASES:
        cfg = sharpened(CONFIGS[name], sharpen)
        folder = str(tmp_path_factory.mktemp(f"vufizen_{name}"))
        tensors = write_model(folder, cfg, seed=11)
        reqs = {f"r{i}": random_tokens(n, cfg["vocab"], 40 + i) for i, n in enumerate(LENGTHS)}
        ref64 = {r: pv.forward(cfg, tensors, t) for r, t in reqs.items()}
        ref = {r: v.numpy().astype(np.float32) for r, v in ref64.items()}
        scale = max(float(v.abs().max()) for v in ref64.values())
        # what rounding alone does at every position: the plain implementation in 32-bit against itself in 64-bit
        # (the largest so far at every position: what a request carries is rounded on and on, and one position's error is one draw)
        NOISE[(name, sharpen)] = {r: np.maximum.accumulate(((pv.forward(cfg, tensors, t, dtype=torch.float32).double() - ref64[r])
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
        rounded = {r: pv.forward(cfg, tensors, t, dtype=torch.bfloat16).float().numpy() for r, t in some.items()}
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
    """A lost convolution tap, a state that is not carried, a map that is left out, a gate without its bias: each moves the
    logits by far more than any tolerance above."""
    folder, cfg, tensors, reqs, ref = models[case]
    toks = reqs["r7"]
    scale = float(np.abs(ref["r7"]).max())

    def moved(**other):
        w = dict(tensors, **{k.replace("__", "."): v for k, v in other.items()})
        return float(np.abs(pv.forward(cfg, w, toks).numpy() - ref["r7"]).max()) / scale

    allowed = 100 * max(TOL_F32, float(NOISE[case]["r7"].max()))
    oldest = tensors["l0.mix.k.conv"].clone()
    oldest[:, 0] = 0
    assert moved(l0__mix__k__conv=oldest) > allowed
    assert moved(l1__mix__f=torch.zeros_like(tensors["l1.mix.f"])) > allowed
    assert moved(l0__mix__lq1=torch.zeros_like(tensors["l0.mix.lq1"])) > allowed
    assert moved(l0__rg1__b=torch.zeros_like(tensors["l0.rg1.b"])) > allowed
    assert moved(l1__norm1=2.0 * tensors["l1.norm1"]) > allowed


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
            toks.append(int(pv.forward(cfg, tensors, toks)[-1].argmax()))
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
    from inferrs_amd.config.vufizen import VufizenConfig
    from inferrs_amd.engine import Engine
    from inferrs_amd.engine.engine import Entry
    eng = Engine.from_random(VufizenConfig.from_dict(CONFIGS["A"]), seed=1, dtype="bfloat16", page_size=16, num_pages=16, max_seqs=2)
    logits = eng.step([Entry("a", random_tokens(33, 211, 1), [32]), Entry("b", [5], [0])])
    assert logits.shape == (2, 211) and bool(torch.isfinite(logits).all())


def test_command_line_run_and_bench(models):
    """The command line serves the design as it serves the others: greedy tokens are the plain implementation's, a drawn run
    and the timing command finish."""
    folder, cfg, tensors, reqs, ref = models[("A", 1.0)]
    prompt = random_tokens(9, cfg["vocab"], 3)
    toks = list(prompt)
    for _ in range(6):
        toks.append(int(pv.forward(cfg, tensors, toks)[-1].argmax()))
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
