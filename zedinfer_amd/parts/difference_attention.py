"""Attention whose heads are the difference of two softmax maps over the same values."""
from __future__ import annotations

import math
from typing import Dict

import torch

from .. import ops
from ..config.forward_config import PartSpec
from ..weights.loader import WeightSpec
from .base import LayerMemory, Mixer, POSITION_ENCODINGS, Runtime, register_mixer
from .mixers import Attention, LONG_TILE, attention_planner


@register_mixer("difference_attention")
class DifferenceAttention(Attention):
    """Causal grouped-query attention; head h = n(A1 v - lam A2 v) * sigmoid(W_g x)_h, with two softmax maps A1, A2 over the
    same values, each from a query and a key of its own, one number lam = exp(lq1 . lk1) - exp(lq2 . lk2) + ``diff`` for the
    layer, and n(o) = o / sqrt(mean(o^2) + eps) * (1 - diff) over the head's values.  Queries and keys (``head_dim`` values a
    map; rows [head][map]) are RMS-normed per head and map with one gain each, then turned (the position encoding must hand over
    a table of split-half angles, or do nothing); scores are (q . k) * ``scale`` over all earlier positions, or a window.

    The maps are heads of the engine's attention kernels: 2 * num_heads query heads over num_kv_heads cached heads whose key
    row holds both maps' keys side by side, beside one value row.  A query row is zero outside its map's half, so the product
    with the whole key row is its map's score and nothing is cached twice; the prompt kernel for heads of 64 and 128 multiplies
    a map's half alone.  Cached heads hold ``d`` = max(2 head_dim, value_dim) values (in bfloat16 up to 128 rounded up to
    what the matrix-core kernels take), zeros behind what is shorter.  For decoded tokens the kernel that merges a token's
    chunks of keys makes the difference, the norm and the gate as well.

    q, k, v and the gate are one product.  params: hidden_size, num_heads, num_kv_heads, head_dim, value_dim, scale, diff,
    eps, window (0), position, qk_norm (True), gate (True)."""

    graph_safe = True
    tape_safe = True
    padding_safe = True
    maps = 2

    @staticmethod
    def weight_specs(spec: PartSpec) -> Dict[str, WeightSpec]:
        p = spec.params
        H, nh, nkv, d, dv = (int(p[k]) for k in ("hidden_size", "num_heads", "num_kv_heads", "head_dim", "value_dim"))
        w = {"q": WeightSpec((nh * 2 * d, H)), "k": WeightSpec((nkv * 2 * d, H)), "v": WeightSpec((nkv * dv, H)),
             "o": WeightSpec((H, nh * dv))}
        w.update({x: WeightSpec((d,)) for x in ("lq1", "lk1", "lq2", "lk2")})
        if p.get("qk_norm", True):
            w.update({"q_norm": WeightSpec((d,), init="ones"), "k_norm": WeightSpec((d,), init="ones")})
        if p.get("gate", True):
            w["g"] = WeightSpec((nh, H))
        return w

    def __init__(self, spec: PartSpec, weights: Dict[str, torch.Tensor], rt: Runtime):
        Mixer.__init__(self, spec, weights, rt)
        p = spec.params
        self.hidden = int(p["hidden_size"])
        self.heads, self.nkv, self.dim, self.vdim = (int(p[k]) for k in ("num_heads", "num_kv_heads", "head_dim", "value_dim"))
        if self.heads % self.nkv:
            raise ValueError(f"difference_attention: {self.heads} heads are not a multiple of {self.nkv} key/value heads")
        self.nh = 2 * self.heads                 # of the attention kernels
        big = max(2 * self.dim, self.vdim)
        self.d = -(-big // 16) * 16 if (rt.dtype == torch.bfloat16 and big <= 128) else -(-big // 2) * 2
        self.qd = self.nh * self.d
        self.window = int(p.get("window", 0) or 0)
        self.scale, self.eps = float(p["scale"]), float(p["eps"])
        pos_spec: PartSpec = p["position"]
        self.position = POSITION_ENCODINGS.get(pos_spec.kind)(pos_spec, {}, rt)
        diff = float(p["diff"])
        l1, l2 = (float((weights["lq" + i].double() * weights["lk" + i].double()).sum()) for i in ("1", "2"))
        self.lam, self.factor = math.exp(l1) - math.exp(l2) + diff, 1.0 - diff
        mats = [weights["q"], weights["k"], weights["v"]]
        self.width = sum(int(m.shape[0]) for m in mats)
        self.gated = bool(p.get("gate", True))
        if self.gated:
            mats.append(weights["g"])
        rows = sum(int(m.shape[0]) for m in mats)
        if rows % 8:                             # rows of the product to a multiple of 8
            mats.append(torch.zeros((-rows % 8, self.hidden), dtype=mats[0].dtype, device=mats[0].device))
        self.qkvg = torch.cat([m.to(mats[0].dtype) for m in mats]).contiguous()
        self.q_gain = self.k_gain = None
        if p.get("qk_norm", True):
            self.q_gain, self.k_gain = weights["q_norm"].float().contiguous(), weights["k_norm"].float().contiguous()
        self.o = weights["o"]
        self.qk_norm = False                     # (of the base class: its own way)
        self.wide_tile = ops.attention_prefill_tile(rt.dtype, self.d) if rt.device.type == "cuda" else LONG_TILE
        self.plan_key = attention_planner(self.wide_tile, self.nh).key

    def tune(self, num_tokens: int) -> None:
        n = int(num_tokens)
        self.rt.tune_linear(self.rt.buffer("norm_out", (n, self.hidden)), self.qkvg)
        self.rt.tune_linear(self.rt.buffer("difference_heads", (n, self.heads * self.vdim)), self.o)

    def forward(self, x: torch.Tensor, batch, memory: LayerMemory) -> torch.Tensor:
        n, rt = x.shape[0], self.rt
        view = batch.groups[memory.group]
        kc, vc = memory.tensors["k"], memory.tensors["v"]
        table = self.position.step_table(batch)
        if table is None:
            raise ValueError("difference_attention: the position encoding must hand over a table of split-half angles")
        rows = self.qkvg.shape[0]
        if ops.linear_sums_supported(x, self.qkvg):
            # few rows: the kernels that read the projection add its partial sums
            S = ops.linear_splits(n, rows, self.hidden)
            full = ops.linear_sums(x, self.qkvg, out=rt.buffer("difference_proj_sums", (S, n, rows), torch.float32))
        else:
            full = ops.linear(x, self.qkvg, out=rt.buffer("difference_proj", (n, rows)))
        gate = full[..., self.width:self.width + self.heads] if self.gated else None
        writes, plan = memory.writes, batch.plans[self.plan_key]
        # the rest of the query rows is zeroed unless nobody reads it
        pad = plan.sizes["num_short"] > 0 or not self.prompt_reads_parts(rt.dtype, kc.shape[2])
        q = rt.buffer("attn_q", (n, self.qd))
        ops.head_norm_store(full[..., :self.width], self.q_gain, self.k_gain, self.eps, None if isinstance(table, str) else table,
                            view.slots if writes else None, kc if writes else None, vc if writes else None, self.heads, self.nkv,
                            self.maps, self.dim, self.vdim, self.d, q_out=q, pad=pad)
        heads = rt.buffer("difference_heads", (n, self.heads * self.vdim))
        constants = (self.lam, self.factor, self.eps)
        if batch.single_tokens and ops.attention_decode_supported(q.dtype, self.nh, self.nkv, self.d, kc.shape[2]):
            max_keys = plan.sizes["max_short_keys"]
            ws = rt.buffer("attn_split", (ops.attention_decode_workspace(n, self.nh, self.d),), torch.float32)
            ops.attention_decode(q, kc, vc, batch.tok_seq, batch.positions, view.block_tables, self.nh, self.nkv, self.d, self.scale,
                                 max_keys, self.window, workspace=ws, leave_chunks=True)
            ops.difference_merge(ws, batch.positions, self.heads, self.d, self.vdim, max_keys, *constants, out=heads, gate=gate,
                                 window=self.window)
            return self.project(heads, n)
        att = rt.buffer("attn_out", (n, self.qd))
        self.attend(q, att, batch, view, memory)
        ops.difference_heads(att, self.heads, self.d, self.vdim, *constants, out=heads, gate=gate)
        return self.project(heads, n)

    def project(self, att: torch.Tensor, n: int) -> torch.Tensor:
        if ops.linear_sums_supported(att, self.o):
            S = ops.linear_splits(n, self.hidden, self.o.shape[1])
            return ops.linear_sums(att, self.o, out=self.rt.buffer("attn_proj_sums", (S, n, self.hidden), torch.float32))
        return ops.linear(att, self.o, out=self.rt.buffer("attn_proj", (n, self.hidden)))
