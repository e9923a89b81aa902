"""Checked launches of the kernels behind several residual streams a token, behind attention whose heads are differences
of two softmax maps, and an activation alone or in a product's epilogue."""
from __future__ import annotations

from ctypes import c_void_p
from typing import Optional

import torch

from . import _lib
from .functional import BF16, F32, FEW_ROWS, _angle_table, _check_cache, _code, _few_rows_operands, _gpu, _i32, _p, _rows, _stream, attention_decode_workspace
from .mixing import _f32
from .sublayers import _terms

ACTIVATIONS = {"silu": 0, "gelu_tanh": 1, "gelu_erf": 2, "relu2": 3}


def stream_mix_max_streams() -> int:
    return int(_lib.load().zi_stream_mix_max_streams())


def stream_mix(streams: torch.Tensor, read: torch.Tensor, gain: torch.Tensor, eps: float, centered: bool, out: torch.Tensor,
               y: Optional[torch.Tensor] = None, write: Optional[torch.Tensor] = None, scale: Optional[torch.Tensor] = None,
               keep: Optional[torch.Tensor] = None, rows: Optional[torch.Tensor] = None) -> torch.Tensor:
    """``streams`` float32 [s, n, H], or [n, H] when all of them are equal (then ``read`` tells how many).  With ``y`` ([n, H],
    or a stack [S, n, H] of float32 terms): X_t <- sum_s write[s, t] X_s + write[s * s + t] (y * scale), ``write`` float32
    [s * s + s], ``scale`` float32 [H] or None (ones).  ``keep`` float32 [s, n, H] (may be ``streams``) receives the new
    streams.  out [m, H] = the norm (``gain`` float32 [H]; ``centered``: a layer norm, else an RMS norm) of
    sum_t read[t] X_t, ``read`` float32 [s].  ``rows`` int32 [m] picks the rows that are made (then nothing is kept)."""
    _gpu("stream_mix", streams, read, gain, out, y, write, scale, keep, rows)
    s = int(read.numel())
    _f32(read, "stream_mix read", (s,))
    if streams.dtype != torch.float32 or not streams.is_contiguous() or streams.dim() not in (2, 3) \
            or (streams.dim() == 3 and streams.shape[0] != s):
        raise ValueError(f"stream_mix: the streams must be contiguous float32 [{s}, n, H], or [n, H] for equal ones")
    n, H = int(streams.shape[-2]), int(streams.shape[-1])
    _f32(gain, "stream_mix gain", (H,))
    splits, stride, y_code = 1, 0, F32
    if y is not None:
        if not y.is_contiguous() or tuple(y.shape[-2:]) != (n, H):
            raise ValueError(f"stream_mix: y must be a contiguous [{n}, {H}] tensor or a stack of such")
        splits, stride = _terms(y, "stream_mix y")[:2]
        y_code = _code(y, "stream_mix y")
        _f32(write, "stream_mix write", (s * s + s,))
        if scale is not None:
            _f32(scale, "stream_mix scale", (H,))
    if keep is not None:
        if y is None or rows is not None:
            raise ValueError("stream_mix: streams are kept where a result is written into all rows")
        _f32(keep, "stream_mix keep", (s, n, H))
    m = n
    if rows is not None:
        _i32(rows, "stream_mix rows")
        m = int(rows.numel())
    if tuple(out.shape) != (m, H) or not out.is_contiguous():
        raise ValueError(f"stream_mix: out must be a contiguous [{m}, {H}] tensor")
    _lib.call("zi_stream_mix", _p(out), _code(out, "stream_mix out"), _p(streams), n * H if streams.dim() == 3 else 0, _p(keep),
              n * H if keep is not None else 0, _p(y), y_code, splits, stride, _p(scale if y is not None else None),
              _p(write if y is not None else None), _p(read), _p(gain), _p(rows), m, n, s, H, float(eps), int(bool(centered)), _stream())
    return out


def head_norm_store(proj: torch.Tensor, q_gain: Optional[torch.Tensor], k_gain: Optional[torch.Tensor], eps: float,
                    table: Optional[torch.Tensor], slots: Optional[torch.Tensor], kcache: Optional[torch.Tensor],
                    vcache: Optional[torch.Tensor], nh: int, nkv: int, maps: int, dim: int, vdim: int, d: int,
                    q_out: torch.Tensor, pad: bool = True) -> torch.Tensor:
    """proj [n, q | k | v] (any storage type, dense rows; or a stack of float32 partial sums): q holds nh heads of ``maps``
    queries of ``dim`` values, k as many keys for each of nkv heads, v one value of ``vdim`` values each.  Every query and key
    is RMS-normed with its gain (float32 [dim], or None) and its first R dims turn as split halves by ``table`` [n, R/2, 2].
    Queries go to ``q_out`` [n, nh * maps * d], map m's into the m-th of the row's ``maps`` parts (``pad``: the rest of the row
    becomes zero, else it is not written); keys and values of tokens with a slot into the caches, whose heads hold ``d`` values
    (a head's keys side by side in one row, zeros behind what is shorter)."""
    _gpu("head_norm_store", proj, q_gain, k_gain, table, slots, kcache, vcache, q_out)
    splits, split_stride, ld, n, width = _terms(proj, "head_norm_store proj", columns=True)
    if width != (nh + nkv) * maps * dim + nkv * vdim:
        raise ValueError(f"head_norm_store: proj must be [n, {(nh + nkv) * maps * dim + nkv * vdim}]")
    for name, g in (("q_gain", q_gain), ("k_gain", k_gain)):
        if g is not None:
            _f32(g, f"head_norm_store {name}", (dim,))
    rot = _angle_table(table, n, dim, "head_norm_store")
    ldq, wq = _rows(q_out, "head_norm_store q_out")
    if tuple(q_out.shape) != (n, nh * maps * d):
        raise ValueError(f"head_norm_store: q_out must be [n, {nh * maps * d}]")
    pages = ps = 0
    if kcache is not None:
        if slots is None:
            raise ValueError("head_norm_store: a cache needs the tokens' slots")
        pages, ps = _check_cache(kcache, vcache, nkv, d, q_out.dtype, "head_norm_store")
        _i32(slots, "head_norm_store slots", n)
    _lib.call("zi_head_norm_store", _p(q_out), _code(q_out, "head_norm_store q_out"), ldq, _p(kcache),
              _p(vcache if kcache is not None else None), _p(proj), _code(proj, "head_norm_store proj"), ld, splits, split_stride,
              _p(q_gain), _p(k_gain), float(eps), _p(table), rot, _p(slots if kcache is not None else None), pages * ps, n, nh, nkv,
              maps, dim, vdim, d, max(ps, 1), int(bool(pad)), _stream())
    return q_out


def _head_gate(gate: Optional[torch.Tensor], n: int, heads: int, what: str):
    """(gate, type code, row stride, terms, stride between terms) of one number a head and token, or a stack of terms of it."""
    if gate is None:
        return _p(None), F32, 0, 1, 0
    if gate.dim() not in (2, 3) or tuple(gate.shape[-2:]) != (n, heads) or gate.stride(-1) != 1 \
            or (gate.dim() == 3 and gate.dtype != torch.float32):
        raise ValueError(f"{what}: the gate must be [{n}, {heads}] or a float32 stack of such rows")
    stack = gate.dim() == 3
    return _p(gate), _code(gate, what), int(gate.stride(-2)), int(gate.shape[0]) if stack else 1, int(gate.stride(0)) if stack else 0


def difference_heads(att: torch.Tensor, heads: int, d: int, vdim: int, lam: float, factor: float, eps: float, out: torch.Tensor,
                     gate: Optional[torch.Tensor] = None) -> torch.Tensor:
    """att [n, heads * 2 * d]: two maps' attention a head; out [n, heads * vdim] = o / sqrt(mean(o^2) + eps) * factor *
    sigmoid(gate), o = (first ``vdim`` values of map 1) - lam * (of map 2); gate [n, heads] (or a stack of terms) or None."""
    _gpu("difference_heads", att, out, gate)
    lda, wa = _rows(att, "difference_heads att")
    ldo, wo = _rows(out, "difference_heads out")
    n = att.shape[0]
    if wa != 2 * heads * d or tuple(out.shape) != (n, heads * vdim) or out.dtype != att.dtype:
        raise ValueError(f"difference_heads: att must be [n, {2 * heads * d}] and out [n, {heads * vdim}] of one type")
    _lib.call("zi_difference_heads", _p(out), _code(out, "difference_heads out"), ldo, _p(att), lda, n, heads, d, vdim, float(lam),
              float(factor), float(eps), *_head_gate(gate, n, heads, "difference_heads"), _stream())
    return out


def difference_merge(workspace: torch.Tensor, tok_pos: torch.Tensor, heads: int, d: int, vdim: int, max_keys: int, lam: float,
                     factor: float, eps: float, out: torch.Tensor, gate: Optional[torch.Tensor] = None, window: int = 0) -> torch.Tensor:
    """``difference_heads`` straight from the chunks that ``attention_decode(..., leave_chunks=True)`` left in ``workspace`` for
    2 * heads heads of ``d`` values (same tokens, ``max_keys`` and ``window``); out bfloat16 [n, heads * vdim]."""
    _gpu("difference_merge", workspace, tok_pos, out, gate)
    n = tok_pos.numel()
    _i32(tok_pos, "difference_merge tok_pos", n)
    ldo, wo = _rows(out, "difference_merge out")
    if tuple(out.shape) != (n, heads * vdim) or out.dtype != torch.bfloat16 or vdim > d:
        raise ValueError(f"difference_merge: out must be bfloat16 [{n}, {heads * vdim}] with heads within {d}")
    need = attention_decode_workspace(n, 2 * heads, d)
    if workspace.dtype != torch.float32 or workspace.numel() < need or not workspace.is_contiguous():
        raise ValueError(f"difference_merge: workspace must be a contiguous float32 buffer of {need} entries")
    if window > 0:
        max_keys = min(max_keys, window)
    _lib.call("zi_difference_merge", _p(out), ldo, _p(workspace), workspace.numel(), n, _p(tok_pos), int(window),
              int(_lib.load().zi_attention_decode_chunks(int(max_keys))), heads, d, vdim, float(lam), float(factor), float(eps),
              *_head_gate(gate, n, heads, "difference_merge"), _stream())
    return out


def activate(z: torch.Tensor, activation: str, out: torch.Tensor) -> torch.Tensor:
    """out [n, I] = act(z): "silu", "gelu_tanh", "gelu_erf" or "relu2" (relu squared); z [n, I] with dense rows or a stack
    [S, n, I] of float32 partial sums."""
    _gpu("activate", z, out)
    splits, split_stride, ldz, n, I = _terms(z, "activate z")
    ldo, Io = _rows(out, "activate out")
    if tuple(out.shape) != (n, I):
        raise ValueError("activate: out has the wrong shape")
    if activation not in ACTIVATIONS:
        raise ValueError(f"activate: unknown activation {activation!r}")
    _lib.call("zi_activate", _p(out), _code(out, "activate out"), ldo, _p(z), _code(z, "activate z"), ldz, splits, split_stride, n, I,
              ACTIVATIONS[activation], _stream())
    return out


def linear_activated_supported(x: torch.Tensor, weight: torch.Tensor, activation: str) -> bool:
    """Whether ``linear_activated`` takes the operands and is no slower than a product that may be cut and ``activate``."""
    return (activation in ACTIVATIONS and activation != "gelu_erf" and _few_rows_operands(x, weight, FEW_ROWS)
            and bool(_lib.load().zi_gemm_skinny_act_pays(int(x.shape[0]), int(weight.shape[0]), int(weight.shape[1]))))


def linear_activated(x: torch.Tensor, weight: torch.Tensor, activation: str, bias: Optional[torch.Tensor] = None,
                     out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """act(x . weight^T + bias) in one kernel for few rows, bfloat16 [M, N]: ``ACTIVATIONS`` but the error function's."""
    _gpu("linear_activated", x, weight, bias, out)
    if activation not in ACTIVATIONS or activation == "gelu_erf":
        raise ValueError(f"linear_activated: no activation {activation!r} in this product")
    if not _few_rows_operands(x, weight, FEW_ROWS):
        raise ValueError(f"linear_activated: needs bfloat16 operands of at most {FEW_ROWS} rows, K and row strides multiples of 8")
    (M, K), N = x.shape, weight.shape[0]
    if bias is not None and (bias.dtype != torch.bfloat16 or bias.numel() != N or not bias.is_contiguous()):
        raise ValueError(f"linear_activated: the bias must be a contiguous bfloat16 [{N}] tensor")
    if out is None:
        out = torch.empty((M, N), dtype=torch.bfloat16, device=x.device)
    ldo, _ = _rows(out, "linear_activated out")
    if tuple(out.shape) != (M, N) or out.dtype != torch.bfloat16:
        raise ValueError(f"linear_activated: out must be bfloat16 [{M}, {N}]")
    _lib.call("zi_gemm_skinny_act", _p(out), BF16, 4 + ACTIVATIONS[activation], _p(x), _p(weight), _p(bias), M, N, K, x.stride(0),
              weight.stride(0), ldo, c_void_p(0), 0, 0.0, _stream())
    return out
