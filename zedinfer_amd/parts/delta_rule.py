"""The gated delta rule: a recurrent mixer with a matrix state per head."""
from __future__ import annotations

from typing import Dict, Optional

import torch

from .. import ops
from ..config.forward_config import PartSpec
from ..weights.loader import WeightSpec
from .base import LayerMemory, Mixer, Runtime, StateRequest, register_mixer
from .rows import ProductRows


@register_mixer("gated_delta_rule")
class GatedDeltaRule(Mixer):
    """Per head a state S [dim, vdim] (float32, zero at a sequence's start), updated token by token:

        S <- g S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q      (the read-out sees the token's write)

    q and k [kv_heads, dim] and v [heads, vdim] are projections of x that pass a short causal convolution over
    time (per channel, ``conv`` taps, no bias, zeros before the start) and SiLU; q and k are then made unit vectors
    per head (x / sqrt(sum x^2 + 1e-6)), q also times dim^-1/2; head h reads q/k head h // (heads / kv_heads).
    beta = sigmoid(W_b x) and the decay g = exp(-exp(A_log) softplus(W_a x + dt_bias)), one of each per head.
    The output per head is o / rms(o) * w [vdim] * silu(W_g x), then W_o.

    A request's state is S and the last conv - 1 rows that entered the convolution, in one float32 row of the
    state slot.  The six projections are one stacked product with float32 results; everything after it up to the
    output projection is float32 arithmetic (``csrc/delta.hip``).  Steps of such a model are never padded.

    params: hidden_size, heads, kv_heads, dim, vdim, conv, eps."""

    graph_safe = True
    tape_safe = True
    padding_safe = False      # a padding token would move the state
    writes_into = True

    @staticmethod
    def weight_specs(spec: PartSpec) -> Dict[str, WeightSpec]:
        p = spec.params
        H, nh, kvh, dim, vdim, taps = (int(p[k]) for k in ("hidden_size", "heads", "kv_heads", "dim", "vdim", "conv"))
        return {"q": WeightSpec((kvh * dim, H)), "q_conv": WeightSpec((kvh * dim, taps)),
                "k": WeightSpec((kvh * dim, H)), "k_conv": WeightSpec((kvh * dim, taps)),
                "v": WeightSpec((nh * vdim, H)), "v_conv": WeightSpec((nh * vdim, taps)),
                "b": WeightSpec((nh, H)), "a": WeightSpec((nh, H)), "A_log": WeightSpec((nh,), init="zeros"),
                "dt_bias": WeightSpec((nh,), init="zeros"), "norm": WeightSpec((vdim,), init="ones"),
                "g": WeightSpec((nh * vdim, H)), "o": WeightSpec((H, nh * vdim))}

    def __init__(self, spec: PartSpec, weights: Dict[str, torch.Tensor], rt: Runtime):
        super().__init__(spec, weights, rt)
        p = spec.params
        self.hidden, self.nh, self.kvh, self.dim, self.vdim, self.taps = (
            int(p[k]) for k in ("hidden_size", "heads", "kv_heads", "dim", "vdim", "conv"))
        self.eps = float(p.get("eps", 1e-6))
        if self.nh % self.kvh:
            raise ValueError(f"gated_delta_rule: {self.nh} heads are not a multiple of {self.kvh} q/k heads")
        if not (1 <= self.taps <= ops.mixing.DELTA_MAX_TAPS) or self.dim > 256:
            raise ValueError("gated_delta_rule: conv must lie in 1..17 and dim be at most 256")
        self.channels = 2 * self.kvh * self.dim + self.nh * self.vdim
        self.gate_at = self.channels
        width = self.channels + self.nh * self.vdim + 2 * self.nh
        mats = [weights[k] for k in ("q", "k", "v", "g", "b", "a")]
        dt = mats[0].dtype
        stacked = torch.zeros((-(-width // 8) * 8, self.hidden), dtype=dt, device=mats[0].device)   # rows to a multiple of 8
        at = 0
        for m in mats:
            stacked[at:at + m.shape[0]] = m.to(dt)
            at += m.shape[0]
        self.w_in = stacked
        self.width = width
        self.conv_w = torch.cat([weights[k].float() for k in ("q_conv", "k_conv", "v_conv")]).contiguous()
        self.a_log, self.dt_bias = weights["A_log"].float().contiguous(), weights["dt_bias"].float().contiguous()
        self.norm = weights["norm"].float().contiguous()
        self.o = weights["o"]

    def state_request(self) -> Optional[StateRequest]:
        return StateRequest((ops.delta_state_floats(self.nh, self.dim, self.vdim, self.kvh, self.taps),), torch.float32)

    def step_rows(self, rows: int, kind: str) -> int:
        return ProductRows.step_rows(rows, kind)

    def forward(self, x: torch.Tensor, batch, memory: LayerMemory, out=None) -> torch.Tensor:
        n, rt, nh, kvh, dim, vdim = x.shape[0], self.rt, self.nh, self.kvh, self.dim, self.vdim
        state = memory.state
        full = ops.linear(x, self.w_in, out=rt.buffer("delta_proj", (n, self.w_in.shape[0]), torch.float32))
        proj = full[:, :self.width]
        qk = rt.buffer("delta_qk", (n, 2 * kvh * dim), torch.float32)
        v = rt.buffer("delta_v", (n, nh * vdim), torch.float32)
        beta_g = rt.buffer("delta_beta_g", (n, 2, nh), torch.float32)
        ops.delta_prepare(proj, self.conv_w, self.a_log, self.dt_bias, state, batch.tok_seq, batch.entry_start,
                          batch.entry_slot, nh, kvh, dim, vdim, self.taps, qk, v, beta_g)
        ops.delta_conv_state(state, proj, batch.entry_start, batch.entry_len, batch.entry_slot, nh, kvh, dim, vdim,
                             self.taps)
        o = rt.buffer("delta_read", (n, nh * vdim), torch.float32)
        ops.delta_rule(qk, v, beta_g, state, batch.entry_start, batch.entry_len, batch.entry_slot, nh, kvh, dim, vdim, out=o)
        y = rt.buffer("delta_heads", (n, nh * vdim))
        ops.gated_rms_norm(o, self.norm, proj[:, self.gate_at:self.gate_at + nh * vdim], nh, vdim, self.eps, out=y)
        if out is None:
            out = rt.buffer("delta_out", (n, self.hidden))
        return ops.linear(y, self.o, out=out)


@register_mixer("channel_delta_rule")
class ChannelDeltaRule(Mixer):
    """The delta rule with a decay per key channel: per head a state S [dim, vdim] (float32, zero at a sequence's start),

        S <- diag(g) S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q   (the read-out sees the token's write)

    q, k, v and beta as in ``gated_delta_rule``; the decay comes from a low-rank projection, g = exp(-exp(A_log_h)
    softplus(W_a2 (W_a1 x) + dt_bias)) [heads, dim], and so does the output's gate: o / rms(o) * w [vdim] * sigmoid(W_g2
    (W_g1 x)), then W_o.  The two ranks are the checkpoint's own unless the params name them.

    A request's state is S and the last conv - 1 rows that entered the convolution, in one float32 row of the state
    slot.  q | k | v | b | a1 | g1 are one stacked product with float32 results (each of the two low-rank parts padded to
    a multiple of 32 rows, which the second products read on the matrix cores); everything after it up to the output
    projection is float32 arithmetic (``csrc/delta.hip``, ``csrc/delta_channel.hip``).  Steps of such a model are never
    padded.

    params: hidden_size, heads, kv_heads, dim, vdim, conv, eps, decay_rank (-1), gate_rank (-1)."""

    graph_safe = True
    tape_safe = True
    padding_safe = False      # a padding token would move the state
    RANK_ROWS = 32

    @staticmethod
    def weight_specs(spec: PartSpec) -> Dict[str, WeightSpec]:
        p = spec.params
        H, nh, kvh, dim, vdim, taps = (int(p[k]) for k in ("hidden_size", "heads", "kv_heads", "dim", "vdim", "conv"))
        ra, rg = int(p.get("decay_rank", -1)), int(p.get("gate_rank", -1))
        return {"q": WeightSpec((kvh * dim, H)), "q_conv": WeightSpec((kvh * dim, taps)),
                "k": WeightSpec((kvh * dim, H)), "k_conv": WeightSpec((kvh * dim, taps)),
                "v": WeightSpec((nh * vdim, H)), "v_conv": WeightSpec((nh * vdim, taps)),
                "b": WeightSpec((nh, H)), "A_log": WeightSpec((nh,), init="zeros"),
                "a1": WeightSpec((ra, H)), "a2": WeightSpec((nh * dim, ra)), "dt_bias": WeightSpec((nh * dim,), init="zeros"),
                "g1": WeightSpec((rg, H)), "g2": WeightSpec((nh * vdim, rg)),
                "norm": WeightSpec((vdim,), init="ones"), "o": WeightSpec((H, nh * vdim))}

    def __init__(self, spec: PartSpec, weights: Dict[str, torch.Tensor], rt: Runtime):
        super().__init__(spec, weights, rt)
        p = spec.params
        self.hidden, self.nh, self.kvh, self.dim, self.vdim, self.taps = (
            int(p[k]) for k in ("hidden_size", "heads", "kv_heads", "dim", "vdim", "conv"))
        self.eps = float(p.get("eps", 1e-6))
        if self.nh % self.kvh:
            raise ValueError(f"channel_delta_rule: {self.nh} heads are not a multiple of {self.kvh} q/k heads")
        if not (1 <= self.taps <= ops.mixing.DELTA_MAX_TAPS) or self.dim > 256:
            raise ValueError("channel_delta_rule: conv must lie in 1..17 and dim be at most 256")
        for one, two in (("a1", "a2"), ("g1", "g2")):
            if weights[one].shape[0] != weights[two].shape[1]:
                raise ValueError(f"channel_delta_rule: {one} has {weights[one].shape[0]} rows, {two} {weights[two].shape[1]} columns")
        self.channels = 2 * self.kvh * self.dim + self.nh * self.vdim
        q = weights["q"]
        up = lambda n, m: -(-n // m) * m
        rank = {x: up(int(weights[x].shape[0]), self.RANK_ROWS) for x in ("a1", "g1")}
        self.a_at = up(self.channels, 8)
        self.g_at = self.a_at + rank["a1"]
        self.b_at = self.g_at + rank["g1"]
        self.width = up(self.b_at + self.nh, 8)
        stacked = torch.zeros((self.width, self.hidden), dtype=q.dtype, device=q.device)
        at = 0
        for name in ("q", "k", "v"):
            stacked[at:at + weights[name].shape[0]] = weights[name].to(q.dtype)
            at += weights[name].shape[0]
        for name, at in (("a1", self.a_at), ("g1", self.g_at), ("b", self.b_at)):
            stacked[at:at + weights[name].shape[0]] = weights[name].to(q.dtype)
        self.w_in = stacked
        # the second products' columns, padded as the first products' rows are
        self.second = {}
        for one, two in (("a1", "a2"), ("g1", "g2")):
            m = weights[two]
            wide = torch.zeros((m.shape[0], rank[one]), dtype=weights["a2"].dtype, device=m.device)
            wide[:, :m.shape[1]] = m.to(wide.dtype)
            self.second[two] = wide
        self.conv_w = torch.cat([weights[k].float() for k in ("q_conv", "k_conv", "v_conv")]).contiguous()
        self.a_log, self.dt_bias = weights["A_log"].float().contiguous(), weights["dt_bias"].float().contiguous()
        self.norm = weights["norm"].float().contiguous()
        self.o = weights["o"]

    def state_request(self) -> Optional[StateRequest]:
        return StateRequest((ops.channel_state_floats(self.nh, self.dim, self.vdim, self.kvh, self.taps),), torch.float32)

    def step_rows(self, rows: int, kind: str) -> int:
        return ProductRows.step_rows(rows, kind)

    def tune(self, num_tokens: int) -> None:
        n = int(num_tokens)
        self.rt.tune_linear(self.rt.buffer("mixer_in", (n, self.hidden)), self.w_in, out_dtype=torch.float32)
        self.rt.tune_linear(self.rt.buffer("delta_heads", (n, self.nh * self.vdim)), self.o)

    def forward(self, x: torch.Tensor, batch, memory: LayerMemory) -> torch.Tensor:
        n, rt, nh, kvh, dim, vdim = x.shape[0], self.rt, self.nh, self.kvh, self.dim, self.vdim
        state = memory.state
        matrices, tails = state[:, :nh * dim * vdim], state[:, nh * dim * vdim:]
        rest = None
        if ops.linear_sums_supported(x, self.w_in):      # few rows: the kernel that convolves adds the partial sums
            S = ops.linear_splits(n, self.width, self.hidden)
            proj = ops.linear_sums(x, self.w_in, out=rt.buffer("delta_proj_sums", (S, n, self.width), torch.float32))
            rest = gates = rt.buffer("delta_lowrank", (n, self.b_at - self.a_at), torch.float32)
        else:
            proj = ops.linear(x, self.w_in, out=rt.buffer("delta_proj", (n, self.width), torch.float32))
            gates = proj[:, self.a_at:self.b_at]
        qk = rt.buffer("delta_qk", (n, 2 * kvh * dim), torch.float32)
        v = rt.buffer("delta_v", (n, nh * vdim), torch.float32)
        beta = rt.buffer("delta_beta_g", (n, 2, nh), torch.float32)
        ops.channel_inputs(proj, self.conv_w, tails, batch.tok_seq, batch.entry_start, batch.entry_len, batch.entry_slot, nh,
                           kvh, dim, vdim, self.taps, self.b_at, qk, v, beta.view(n, 2 * nh), rest_at=self.a_at, rest=rest)
        decay = rt.buffer("delta_decay", (n, nh * dim), torch.float32)
        gate = rt.buffer("delta_gate", (n, nh * vdim), torch.float32)
        ranks = self.g_at - self.a_at
        ops.lowrank_gates(gates[:, :ranks], self.second["a2"], self.dt_bias, self.a_log, gates[:, ranks:], self.second["g2"],
                          decay, gate)
        o = rt.buffer("delta_read", (n, nh * vdim), torch.float32)
        y, single = rt.buffer("delta_heads", (n, nh * vdim)), bool(batch.single_tokens)
        finish = (y, self.norm, gate, self.eps) if single and ops.delta_channel_finishes(vdim, matrices) else None
        ops.delta_channel(qk, v, beta, decay, matrices, batch.entry_start, batch.entry_len, batch.entry_slot, nh, kvh, dim, vdim,
                          out=o, single_tokens=single, finish=finish)
        if finish is None:
            ops.gated_rms_norm_act(o, self.norm, gate, nh, vdim, self.eps, "sigmoid", out=y)
        if ops.linear_sums_supported(y, self.o):      # few rows: the partial sums go to the norm that follows
            S = ops.linear_splits(n, self.hidden, nh * vdim)
            return ops.linear_sums(y, self.o, out=rt.buffer("delta_out_sums", (S, n, self.hidden), torch.float32))
        return ops.linear(y, self.o, out=rt.buffer("delta_out", (n, self.hidden)))
