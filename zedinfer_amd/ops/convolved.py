"""Checked launches of the kernels behind a convolution over time in front of a mixer (with the norm before it), behind
low-rank gates, and behind the delta rule with a decay per key channel."""
from __future__ import annotations

from typing import Optional

import torch

from . import _lib
from .functional import F32, _code, _gpu, _i32, _p, _rows, _stream
from .mixing import DELTA_MAX_TAPS, _f32, delta_state_floats as channel_state_floats      # the same row: matrices, then the convolution's tail
from .sublayers import CONV_MAX_TAPS, _terms


def _delta_terms(delta: Optional[torch.Tensor], n: int, H: int, what: str):
    """(code, splits, stride between splits) of a pending addition: None, [n, H] or a stack [S, n, H] of float32 terms."""
    if delta is None:
        return F32, 0, 0
    if not delta.is_contiguous() or tuple(delta.shape[-2:]) != (n, H) or delta.dim() not in (2, 3):
        raise ValueError(f"{what}: the addition must be a contiguous [{n}, {H}] or [S, {n}, {H}] tensor")
    splits, stride = _terms(delta, what)[:2]
    return _code(delta, what), splits, stride


def _stream_rows(resid: torch.Tensor, what: str):
    _f32(resid, f"{what} resid")
    if resid.dim() != 2:
        raise ValueError(f"{what}: the residual stream must be [n, hidden]")
    return int(resid.shape[0]), int(resid.shape[1])


def stream_scale(resid: torch.Tensor, delta: Optional[torch.Tensor], eps: float, out: torch.Tensor) -> torch.Tensor:
    """resid (float32, in place) += delta (None, [n, H], or a stack [S, n, H] of float32 terms, added in rising order);
    out [n] float32 = 1 / sqrt(mean(resid^2) + eps) of every row."""
    _gpu("stream_scale", resid, delta, out)
    n, H = _stream_rows(resid, "stream_scale")
    code, splits, stride = _delta_terms(delta, n, H, "stream_scale delta")
    _f32(out, "stream_scale out", (n,))
    if not eps > 0:
        raise ValueError("stream_scale: eps must be positive")
    _lib.call("zi_stream_scale", _p(out), _p(resid), _p(delta), code, splits, stride, n, H, float(eps), _stream())
    return out


def _tail(state: Optional[torch.Tensor], taps: int, H: int, what: str) -> int:
    if not (1 <= taps <= CONV_MAX_TAPS):
        raise ValueError(f"{what}: at most {CONV_MAX_TAPS} taps")
    if state is None:
        if taps > 1:
            raise ValueError(f"{what}: {taps} taps need the rows before a step")
        return 0
    if state.dtype != torch.float32 or state.dim() != 2 or state.stride(1) != 1 or state.shape[1] < (taps - 1) * H:
        raise ValueError(f"{what}: the state must be float32 [slots, >= {(taps - 1) * H}] with dense rows")
    return int(state.stride(0))


def input_conv(x: torch.Tensor, conv_w: torch.Tensor, state: Optional[torch.Tensor], tok_seq: torch.Tensor,
               entry_start: torch.Tensor, entry_len: torch.Tensor, entry_slot: torch.Tensor, out: torch.Tensor,
               scale: Optional[torch.Tensor] = None, gain: Optional[torch.Tensor] = None, gain_add: float = 0.0,
               slots: Optional[torch.Tensor] = None) -> torch.Tensor:
    """out[t] = h_t + sum_j conv_w[j] * h_(t - taps + 1 + j) per channel, zeros before a sequence's start; h = x, or with
    ``scale`` (float32 [n]) x[t] * scale[t] * (gain + gain_add).  ``conv_w`` float32 [taps, H].  Rows before an entry's
    first one come from ``state`` [slots, >= (taps - 1) * H] float32 (a column slice is fine) at the entry's slot, which
    then takes the entry's last taps - 1 rows of h.  With ``slots`` (every token's place in the cache, negative: none;
    such tokens stand behind an entry's own) only an entry's own tokens count for that."""
    _gpu("input_conv", x, conv_w, state, tok_seq, entry_start, entry_len, entry_slot, out, scale, gain, slots)
    ldx, H = _rows(x, "input_conv x")
    ldo, Ho = _rows(out, "input_conv out")
    n = x.shape[0]
    if tuple(out.shape) != (n, H):
        raise ValueError("input_conv: out has the wrong shape")
    _f32(conv_w, "input_conv conv_w")
    if conv_w.dim() != 2 or conv_w.shape[1] != H:
        raise ValueError(f"input_conv: conv_w must be [taps, {H}]")
    taps = int(conv_w.shape[0])
    stride = _tail(state, taps, H, "input_conv")
    if scale is not None:
        _f32(scale, "input_conv scale", (n,))
        if gain is None or gain.numel() != H or not gain.is_contiguous():
            raise ValueError(f"input_conv: a scale comes with a contiguous gain of {H} values")
    _i32(tok_seq, "input_conv tok_seq", n)
    E = entry_start.numel()
    for t in (entry_start, entry_len, entry_slot):
        _i32(t, "input_conv entries", E)
    if slots is not None:
        _i32(slots, "input_conv slots", n)
    _lib.call("zi_input_conv", _p(out), _code(out, "input_conv out"), ldo, _p(x), _code(x, "input_conv x"), ldx, _p(scale),
              _p(gain if scale is not None else None), _code(gain, "input_conv gain") if scale is not None else F32,
              float(gain_add), _p(conv_w), _p(state), stride, _p(tok_seq), _p(entry_start), _p(entry_len), _p(entry_slot),
              _p(slots), n, H, taps, _stream())
    return out


def norm_input_conv_supported(hidden: int, taps: int, delta: Optional[torch.Tensor]) -> bool:
    """Whether ``norm_input_conv`` takes these sizes (else: ``stream_scale``, then ``input_conv``)."""
    splits = 0 if delta is None else (int(delta.shape[0]) if delta.dim() == 3 else 1)
    return bool(_lib.load().zi_norm_input_conv_supported(int(hidden), int(taps), splits))


def norm_input_conv(resid: torch.Tensor, delta: Optional[torch.Tensor], gain: torch.Tensor, gain_add: float, eps: float,
                    conv_w: torch.Tensor, state: Optional[torch.Tensor], tok_seq: torch.Tensor, entry_slot: torch.Tensor,
                    out: torch.Tensor, slots: Optional[torch.Tensor] = None) -> torch.Tensor:
    """``stream_scale`` and ``input_conv`` over the normed stream in one launch, for steps in which every entry brings
    one token: resid += delta, h = resid / rms(resid) * (gain + gain_add), out = h + conv(h), the tails moved on."""
    _gpu("norm_input_conv", resid, delta, gain, conv_w, state, tok_seq, entry_slot, out, slots)
    n, H = _stream_rows(resid, "norm_input_conv")
    code, splits, stride = _delta_terms(delta, n, H, "norm_input_conv delta")
    _f32(conv_w, "norm_input_conv conv_w")
    if conv_w.dim() != 2 or conv_w.shape[1] != H or gain.numel() != H or not gain.is_contiguous():
        raise ValueError(f"norm_input_conv: conv_w must be [taps, {H}], the gain [{H}]")
    taps = int(conv_w.shape[0])
    sstride = _tail(state, taps, H, "norm_input_conv")
    if tuple(out.shape) != (n, H) or not out.is_contiguous():
        raise ValueError("norm_input_conv: out must be contiguous, of the stream's shape")
    _i32(tok_seq, "norm_input_conv tok_seq", n)
    _i32(entry_slot, "norm_input_conv entry_slot")
    if slots is not None:
        _i32(slots, "norm_input_conv slots", n)
    _lib.call("zi_norm_input_conv", _p(out), _code(out, "norm_input_conv out"), _p(resid), _p(delta), code, splits, stride,
              _p(gain), _code(gain, "norm_input_conv gain"), float(gain_add), float(eps), _p(conv_w), _p(state), sstride,
              _p(tok_seq), _p(entry_slot), _p(slots), n, H, taps, _stream())
    return out


def lowrank_gates(u_a: torch.Tensor, w_a: torch.Tensor, bias: torch.Tensor, a_log: torch.Tensor, u_g: torch.Tensor,
                  w_g: torch.Tensor, out_a: torch.Tensor, out_g: torch.Tensor) -> None:
    """Two low-rank projections at once, for float32 rows u_a [n, Ra] and u_g [n, Rg] (columns of one projection):
    out_a [n, Ca] = exp(-exp(a_log) * softplus(u_a . w_a^T + bias)), ``a_log`` [Ca / dim] one number for every ``dim``
    neighbouring channels, and out_g [n, Cg] = u_g . w_g^T.  On the matrix cores when the weights are bfloat16 with ranks
    that are multiples of 32 (then u is split into two bfloat16 parts, so that little of it is lost)."""
    _gpu("lowrank_gates", u_a, w_a, bias, a_log, u_g, w_g, out_a, out_g)
    lda, Ra = _rows(u_a, "lowrank_gates u_a")
    ldg, Rg = _rows(u_g, "lowrank_gates u_g")
    n = u_a.shape[0]
    Ca, Cg = int(w_a.shape[0]), int(w_g.shape[0])
    if u_a.dtype != torch.float32 or u_g.dtype != torch.float32 or u_g.shape[0] != n or (n > 1 and lda != ldg):
        raise ValueError("lowrank_gates: u_a and u_g must be float32 columns of one projection")
    if tuple(w_a.shape) != (Ca, Ra) or tuple(w_g.shape) != (Cg, Rg) or not w_a.is_contiguous() or not w_g.is_contiguous() \
            or w_a.dtype != w_g.dtype:
        raise ValueError("lowrank_gates: the weights must be contiguous [channels, rank] tensors of one type")
    _f32(bias, "lowrank_gates bias", (Ca,))
    _f32(a_log, "lowrank_gates a_log")
    if Ca % a_log.numel():
        raise ValueError("lowrank_gates: the channels must divide evenly over the heads")
    _f32(out_a, "lowrank_gates out_a", (n, Ca))
    _f32(out_g, "lowrank_gates out_g", (n, Cg))
    _lib.call("zi_lowrank_gates", _p(out_a), _p(u_a), _p(w_a), Ca, Ra, _p(bias), _p(a_log), Ca // a_log.numel(), _p(out_g),
              _p(u_g), _p(w_g), Cg, Rg, _code(w_a, "lowrank_gates w"), max(lda, ldg), n, _stream())


def channel_inputs(proj: torch.Tensor, conv_w: torch.Tensor, tails: Optional[torch.Tensor], tok_seq: torch.Tensor,
                   entry_start: torch.Tensor, entry_len: torch.Tensor, entry_slot: torch.Tensor, heads: int, kv_heads: int,
                   dim: int, vdim: int, taps: int, beta_at: int, qk: torch.Tensor, v: torch.Tensor, beta: torch.Tensor,
                   rest_at: int = 0, rest: Optional[torch.Tensor] = None) -> None:
    """From rows proj [n, q | k | v | ...] (float32), or a stack [S, n, ...] of partial sums of them: the short convolution
    (``conv_w`` [channels, taps]) and SiLU of q, k and v, q and k made unit vectors per head (q also times dim^-1/2) into
    ``qk`` [n, 2 kv_heads dim], v into ``v`` [n, heads vdim], beta = sigmoid(b) with b at column ``beta_at`` into the
    first ``heads`` columns of ``beta``'s rows (row stride free); the sums of the columns ``rest_at`` ... into ``rest``
    [n, columns], if given.  Rows before an entry's first one come from ``tails`` [slots, >= (taps - 1) channels] (dense
    rows) at the entry's slot, which then takes the entry's last taps - 1 rows."""
    _gpu("channel_inputs", proj, conv_w, tails, tok_seq, entry_start, entry_len, entry_slot, qk, v, beta, rest)
    splits, split_stride, ld, n, width = _terms(proj, "channel_inputs proj", columns=True)
    C = 2 * kv_heads * dim + heads * vdim
    if proj.dtype != torch.float32 or not (C <= beta_at <= width - heads):
        raise ValueError(f"channel_inputs: proj must be float32 with the {C} channels first and beta behind them")
    _f32(conv_w, "channel_inputs conv_w", (C, taps))
    _f32(qk, "channel_inputs qk", (n, 2 * kv_heads * dim))
    _f32(v, "channel_inputs v", (n, heads * vdim))
    if beta.dtype != torch.float32 or beta.shape[0] != n or beta.stride(-1) != 1 or beta[0].numel() < heads:
        raise ValueError(f"channel_inputs: beta must be float32 [n, >= {heads}]")
    cols = 0
    if rest is not None:
        cols = int(rest.shape[1])
        _f32(rest, "channel_inputs rest", (n, cols))
        if not (C <= rest_at <= width - cols):
            raise ValueError("channel_inputs: the columns to be added up lie outside the rows")
    if not (1 <= taps <= DELTA_MAX_TAPS) or dim > 256:
        raise ValueError(f"channel_inputs: at most {DELTA_MAX_TAPS} taps and heads of 256 channels")
    stride = 0
    if taps > 1:
        if tails is None or tails.dtype != torch.float32 or tails.dim() != 2 or tails.stride(1) != 1 or tails.shape[1] < (taps - 1) * C:
            raise ValueError(f"channel_inputs: tails must be float32 [slots, >= {(taps - 1) * C}] with dense rows")
        stride = int(tails.stride(0))
    _i32(tok_seq, "channel_inputs tok_seq", n)
    E = entry_start.numel()
    for t in (entry_start, entry_len, entry_slot):
        _i32(t, "channel_inputs entries", E)
    _lib.call("zi_channel_inputs", _p(qk), _p(v), _p(beta), int(beta.stride(0)), _p(rest), _p(proj), ld, splits, split_stride,
              _p(conv_w), _p(tails if taps > 1 else None), stride, _p(tok_seq), _p(entry_start), _p(entry_len), _p(entry_slot), n,
              heads, kv_heads, dim, vdim, taps, int(beta_at), int(rest_at), cols, _stream())


def delta_channel_finishes(vdim: int, state: torch.Tensor) -> bool:
    """Whether ``delta_channel`` can norm and gate the read-outs of single tokens itself (``finish``)."""
    return bool(_lib.load().zi_delta_channel_finishes(int(vdim), int(state.stride(0)))) and state.data_ptr() % 16 == 0


def delta_channel(qk: torch.Tensor, v: torch.Tensor, beta_g: torch.Tensor, decay: torch.Tensor, state: torch.Tensor,
                  entry_start: torch.Tensor, entry_len: torch.Tensor, entry_slot: torch.Tensor, heads: int, kv_heads: int,
                  dim: int, vdim: int, out: torch.Tensor, single_tokens: bool = False, finish=None) -> torch.Tensor:
    """Every entry's tokens in order, per head: S <- diag(decay) S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q, with
    S read from and left in ``state`` [slots, >= heads*dim*vdim] float32 (dense rows); qk [n, 2 kv_heads dim] (q, then
    k), v [n, heads vdim], ``beta_g`` [n, 2, heads] (beta first; the rest is not read), decay [n, heads dim], out
    [n, heads vdim], all float32.  ``single_tokens``: every entry brings one token.  ``finish`` (y, norm, gate, eps; only
    then, and where ``delta_channel_finishes``): y [n, heads vdim] = o / rms(o over a head) * norm [vdim] * sigmoid(gate)
    is written instead of o."""
    _gpu("delta_channel", qk, v, beta_g, decay, state, entry_start, entry_len, entry_slot, out)
    n = qk.shape[0]
    _f32(qk, "delta_channel qk", (n, 2 * kv_heads * dim))
    _f32(v, "delta_channel v", (n, heads * vdim))
    _f32(beta_g, "delta_channel beta_g", (n, 2, heads))
    _f32(decay, "delta_channel decay", (n, heads * dim))
    _f32(out, "delta_channel out", (n, heads * vdim))
    if state.dtype != torch.float32 or state.dim() != 2 or state.stride(1) != 1 or state.shape[1] < heads * dim * vdim:
        raise ValueError(f"delta_channel: the state must be float32 [slots, >= {heads * dim * vdim}] with dense rows")
    if dim > 256:
        raise ValueError(f"delta_channel: dim {dim} is more than the kernel's 256")
    last = (_p(None), F32, _p(None), _p(None), 0.0)
    if finish is not None:
        y, norm, gate, eps = finish
        _gpu("delta_channel finish", y, norm, gate)
        if not single_tokens or not delta_channel_finishes(vdim, state):
            raise ValueError("delta_channel: heads are finished in steps of single tokens, where the kernel holds them whole")
        if tuple(y.shape) != (n, heads * vdim) or not y.is_contiguous():
            raise ValueError("delta_channel: y must be contiguous [n, heads * vdim]")
        _f32(norm, "delta_channel norm", (vdim,))
        _f32(gate, "delta_channel gate", (n, heads * vdim))
        last = (_p(y), _code(y, "delta_channel y"), _p(norm), _p(gate), float(eps))
    E = entry_start.numel()
    for t in (entry_start, entry_len, entry_slot):
        _i32(t, "delta_channel entries", E)
    _lib.call("zi_delta_channel", _p(out), _p(qk), _p(v), _p(beta_g), 2 * heads, _p(decay), _p(state), int(state.stride(0)),
              _p(entry_start), _p(entry_len), _p(entry_slot), E, heads, kv_heads, dim, vdim, int(bool(single_tokens)), *last, _stream())
    return out if finish is None else finish[0]
