"""Python face of the kernels for a stream whose sub-layers are gated and normed before they enter it
(`csrc/gated_branch.hip`), for attention with several maps a head behind a short convolution (`csrc/map_attention.hip`) and
for a matrix state whose rows fade by a gate a channel (`csrc/fading_state.hip`).  Shape checks on the host, then one C
call a kernel; no other implementation stands behind them."""
from __future__ import annotations

import ctypes
from typing import Optional

import torch

from . import KernelError, _DT, _check, _check_cache, _dev, _dt, _f32, _i32, _p, _stream, library
from .mix import MAX_TOP

FADING_MAX_DIM = 512              # rows of a head's matrix that the walk takes
FADING_CHUNK_DIM, FADING_CHUNK_VDIM = 128, 256      # keys and values that the chunks take
FADING_CHUNK = 64                 # tokens of a chunk when long portions run in chunks side by side
FADING_CHUNKS_FROM = 80           # steps whose longest portion has more tokens than this run in chunks (16 heads of 128 x 128: a walk takes
                                  # 10 us and 0.5 us a token, the three kernels of the chunks 45 us up to 128 tokens)
FADING_WORKSPACE_FLOATS = 1 << 28     # a pass over the chunks takes no more than this (1 GiB): more passes beyond


def branch_step(x: torch.Tensor, *, y=None, routed: Optional[torch.Tensor] = None, routed_weights: Optional[torch.Tensor] = None,
                y3=None, y3_scale: Optional[torch.Tensor] = None, gate: Optional[torch.Tensor] = None, gate_off: int = 0,
                gate_bias: Optional[torch.Tensor] = None, weight: torch.Tensor, eps: float,
                x_dtype: Optional[torch.dtype] = None) -> Optional[torch.Tensor]:
    """What closes a sub-layer around a 32-bit stream x [n, width] (changed in place) that sub-layers read as it stands:

        s = y + sum_k routed_weights[:, k] * routed[:, k] + y3_scale[:, None] * y3          (every addend optional)
        s = s * sigmoid(gate[:, gate_off : gate_off + width] + gate_bias)                   (optional; the bias is 32-bit)
        x <- x + rmsnorm(s) * weight

    Returns the new x once more in `x_dtype` (None: nothing).  y and y3 may each be a product still split along its k
    (`Partials`); `routed` [n, top, width] is 32-bit."""
    from . import Partials
    ys = [y, y3]
    if any(isinstance(t, Partials) for t in ys) and any(t is not None and not isinstance(t, Partials) and t.dtype != torch.float32 for t in ys):
        ys = [t.materialize() if isinstance(t, Partials) else t for t in ys]       # (one precision for both)
    splits = [1, 1]
    for i, t in enumerate(ys):
        if isinstance(t, Partials):
            splits[i], ys[i] = t.parts.shape[0], t.parts
    y, y3 = ys
    _dev(x, y, y3, y3_scale, routed, routed_weights, gate_bias, weight)
    for t, name in ((x, "the stream"), (y3_scale, "y3_scale"), (routed, "routed rows"), (routed_weights, "routed weights"),
                    (gate_bias, "gate bias"), (weight, "norm weight")):
        _f32(t, name)
    n, W = x.shape
    given = [t for t in (y, y3) if t is not None]
    for t, sp in ((y, splits[0]), (y3, splits[1])):
        if t is not None and (tuple(t.shape[-2:]) != (n, W) or t.dtype != given[0].dtype or t.dim() not in (2, 3)
                              or (t.dim() == 3 and (t.shape[0] != sp or t.dtype != torch.float32))):
            raise KernelError(f"branch_step: an output {tuple(t.shape)} {t.dtype} does not fit the stream [{n}, {W}]")
    top = 0
    if routed is not None:
        top = routed.shape[1]
        if (routed.dim() != 3 or tuple(routed.shape) != (n, top, W) or top > MAX_TOP or routed_weights is None
                or tuple(routed_weights.shape) != (n, top)):
            raise KernelError(f"branch_step: routed rows {tuple(routed.shape)} and their weights do not fit [{n}, top <= {MAX_TOP}, {W}]")
    if not given and routed is None:
        raise KernelError("branch_step: nothing to add")
    if y3_scale is not None and (y3 is None or y3_scale.numel() != n):
        raise KernelError("branch_step: a factor a row goes with y3 and has one entry a row")
    if weight.numel() != W:
        raise KernelError(f"branch_step: the norm weight has {weight.numel()} entries, the stream is {W} wide")
    g_ld = 0
    if gate is not None:
        if not gate.is_cuda or gate.dim() != 2 or gate.stride(1) != 1 or gate.shape[0] != n or gate_bias is None or gate_bias.numel() != W:
            raise KernelError(f"branch_step: a gate {tuple(gate.shape)} with its bias does not fit the stream [{n}, {W}]")
        g_ld = gate.stride(0) if n > 1 else gate.shape[1]
        if gate_off < 0 or gate_off + W > gate.shape[1]:
            raise KernelError(f"branch_step: a gate of {W} features at {gate_off} of {gate.shape[1]}")
    xr = torch.empty((n, W), dtype=x_dtype, device=x.device) if x_dtype is not None else None
    _check(library().ia_branch_step(
        _p(x), _p(y), _p(y3), splits[0], splits[1], _p(y3_scale), _p(routed), _p(routed_weights), top,
        gate.data_ptr() if gate is not None else None, g_ld, gate_off, _p(gate_bias), _p(weight), ctypes.c_float(eps), _p(xr),
        n, W, _dt(given[0]) if given else 0, _dt(gate) if gate is not None else 0, _DT[x_dtype] if x_dtype is not None else 0, _stream()))
    return xr


# ---- attention with several maps a head --------------------------------------------------------------------------------

def conv_qkv(proj: torch.Tensor, taps: torch.Tensor, state: Optional[torch.Tensor], tail_off: int, *, heads: int, kv_heads: int,
             maps: int, dim: int, vdim: int, q_norm_w: torch.Tensor, k_norm_w: torch.Tensor, eps: float,
             cos: Optional[torch.Tensor], sin: Optional[torch.Tensor], rot: int, interleaved: bool, k_cache: torch.Tensor,
             v_cache: torch.Tensor, slots: torch.Tensor, page_size: int, token_seq: torch.Tensor, cu_tokens: torch.Tensor,
             state_slots: torch.Tensor, max_q_len: int) -> torch.Tensor:
    """From the projections' rows [q: heads x maps x dim | k: kv_heads x maps x dim | v: kv_heads x vdim | ...] to the operands
    of the attention: a causal convolution of `taps` [k, channels] a channel (the last inputs of a request in the [k - 1,
    channels] floats at `tail_off` of its row of `state`), an RMS norm a map of q and k, the turn of each map's first `rot`
    features, the writes of keys [.., maps * dim] and values to their pages.  Returns q [n, heads * maps, maps * dim], a
    map's query zero outside its own part, so that its product with a key head's row is the map's score."""
    _dev(taps, state, q_norm_w, k_norm_w, cos, sin, k_cache, v_cache, slots, token_seq, cu_tokens, state_slots)
    _f32(q_norm_w, "q_norm weight"); _f32(k_norm_w, "k_norm weight"); _f32(cos, "cos"); _f32(sin, "sin"); _f32(state, "state")
    for t, name in ((slots, "slots"), (token_seq, "token_seq"), (cu_tokens, "cu_tokens"), (state_slots, "state_slots")):
        _i32(t, name)
    if not proj.is_cuda or proj.dim() != 2 or not proj.is_contiguous():
        raise KernelError(f"conv_qkv: the projections are contiguous 2-D rows on the GPU, got {tuple(proj.shape)}")
    n, ld = proj.shape
    C = (heads + kv_heads) * maps * dim + kv_heads * vdim
    k = taps.shape[0]
    if tuple(taps.shape) != (k, C) or taps.dtype != proj.dtype or C > ld:
        raise KernelError(f"conv_qkv: taps {tuple(taps.shape)} {taps.dtype} do not fit {C} channels in rows of {ld} {proj.dtype}")
    if k > 1 and (state is None or state.dim() != 2):
        raise KernelError("conv_qkv: the last inputs need a state array [slots, floats a request]")
    if q_norm_w.numel() != dim or k_norm_w.numel() != dim or slots.numel() != n or token_seq.numel() != n:
        raise KernelError("conv_qkv: norm weights of a map's size, a slot and a request a token")
    if cos is not None and (sin is None or tuple(cos.shape) != (n, rot // 2) or sin.shape != cos.shape):
        raise KernelError(f"conv_qkv: rotary tables must be [{n}, {rot // 2}]")
    _check_cache(k_cache, v_cache, kv_heads, page_size, maps * dim, proj.dtype, "conv_qkv", vdim)
    q = torch.empty((n, heads * maps, maps * dim), dtype=proj.dtype, device=proj.device)
    _check(library().ia_conv_qkv(
        _p(q), _p(k_cache), _p(v_cache), _p(proj), ld, _p(taps), k, _p(state), state.shape[1] if state is not None else 0, tail_off,
        _p(q_norm_w), _p(k_norm_w), ctypes.c_float(eps), _p(cos), _p(sin), rot if cos is not None else 0, int(bool(interleaved)),
        _p(slots), _p(token_seq), _p(cu_tokens), _p(state_slots), n, state_slots.numel(), heads, kv_heads, maps, dim, vdim, page_size,
        max(int(max_q_len), 1), _dt(proj), _stream()))
    return q


def differ_norm(a: torch.Tensor, lam: float, eps: float, scale: float) -> torch.Tensor:
    """a [n, 2 H, vdim] (map 1 and map 2 of every head) -> (a1 - lam a2) / sqrt(mean of its squares + eps) * scale, [n, H * vdim]."""
    _dev(a)
    n, rows, dv = a.shape
    if rows % 2:
        raise KernelError(f"differ_norm: two maps a head, got {tuple(a.shape)}")
    out = torch.empty((n, rows // 2 * dv), dtype=a.dtype, device=a.device)
    _check(library().ia_differ_norm(_p(out), _p(a), ctypes.c_float(lam), ctypes.c_float(eps), ctypes.c_float(scale), n, rows // 2, dv,
                                    _dt(a), _stream()))
    return out


# ---- a matrix state whose rows fade by a gate a channel -------------------------------------------------------------------

def fading_scan(proj: torch.Tensor, *, q_off: int, f_off: int, v_off: int, heads: int, dim: int, vdim: int, f_bias: torch.Tensor,
                lower: torch.Tensor, norm_weight: torch.Tensor, eps: float, state: torch.Tensor, s_off: int,
                cu_tokens: torch.Tensor, state_slots: torch.Tensor, max_q_len: int = 0, chunks: Optional[bool] = None) -> torch.Tensor:
    """With u, z and v the slices of proj's rows at q_off, f_off and v_off and f = lower + (1 - lower) sigmoid(z + f_bias) a
    channel: S <- diag(f) S + (1 - f) v^T, o = S^T silu(u) over each request's tokens, from and into the [heads, vdim, dim]
    floats at `s_off` of its state row; returns rmsnorm(o a head) * norm_weight [vdim], [n, heads * vdim] in the precision of
    proj.  `max_q_len`: an upper bound of the tokens a request brings (0: unknown, the step's tokens).  `chunks`: False walks
    every request's tokens in order, True cuts portions into chunks of `FADING_CHUNK` tokens that run side by side (keys up to
    128, values up to 256; differs from the walk by rounding); None: by the longest portion."""
    from .state import group_norm_gate
    _dev(proj, f_bias, lower, norm_weight, state, cu_tokens, state_slots)
    _f32(f_bias, "f_bias"); _f32(lower, "lower"); _f32(norm_weight, "norm weight"); _f32(state, "state")
    _i32(cu_tokens, "cu_tokens"); _i32(state_slots, "state_slots")
    if proj.dim() != 2 or state.dim() != 2:
        raise KernelError("fading_scan: the projections are 2-D rows and the state array [slots, floats a request]")
    n, ld = proj.shape
    if f_bias.numel() != heads * dim or lower.numel() != heads * dim or norm_weight.numel() != vdim:
        raise KernelError(f"fading_scan: gates of {heads} x {dim} channels and a norm over {vdim}")
    if dim > FADING_MAX_DIM:
        raise KernelError(f"fading_scan: a key size of {dim} is beyond {FADING_MAX_DIM}")
    lib = library()
    n_seqs, longest = state_slots.numel(), int(max_q_len) or n
    fits = dim <= FADING_CHUNK_DIM and vdim <= FADING_CHUNK_VDIM
    if chunks is None:
        chunks = fits and longest > FADING_CHUNKS_FROM
    elif chunks and not fits:
        raise KernelError(f"fading_scan: no chunks for keys of {dim} and values of {vdim}")
    count, work = 0, None
    if chunks:
        count = -(-longest // FADING_CHUNK)
        per_chunk = n_seqs * heads * dim * (vdim + 1)
        count = max(1, min(count, FADING_WORKSPACE_FLOATS // per_chunk, 65535 // max(n_seqs, 1)))
        work = torch.empty((lib.ia_fading_scan_workspace(n_seqs, count, heads, dim, vdim),), dtype=torch.float32, device=proj.device)
    out = torch.empty((n, heads * vdim), dtype=proj.dtype if chunks else torch.float32, device=proj.device)
    _check(lib.ia_fading_scan(
        _p(out), _p(state), state.shape[1], s_off, _p(proj), ld, q_off, f_off, v_off, _p(f_bias), _p(lower), _p(norm_weight),
        ctypes.c_float(eps), _p(cu_tokens), _p(state_slots), n_seqs, heads, dim, vdim, max(longest, 1), count, _p(work), _dt(proj),
        _stream()))
    if chunks:
        return out
    return group_norm_gate(out, group=vdim, head=vdim, eps=eps, out_dtype=proj.dtype, weight=norm_weight)
