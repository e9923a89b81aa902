"""A convolution over time in front of any mixer."""
from __future__ import annotations

from dataclasses import replace
from typing import Dict, Optional

import torch

from .. import ops
from ..config.forward_config import PartSpec
from ..weights.loader import WeightSpec
from .base import MIXERS, KVCacheRequest, LayerMemory, Mixer, Part, Runtime, StateRequest, register_mixer
from .norms import RMSNorm


@register_mixer("input_convolution")
class InputConvolution(Mixer):
    """mixer(h + conv(h)): what the mixer reads, the normed stream h, is first replaced by its sum with a causal
    convolution of it over time on each channel, conv(h)_t = sum_j taps[:, j] h_(t - K + 1 + j), zeros before the
    sequence's start.  It stands in front of any registered mixer, whose parameter names appear in this part's weights
    as "mixer.<name>".

    The last K - 1 rows of h are state of the request, in float32, behind the mixer's own state in one row of the slot.
    A block that hands its norm over (``forward_from_stream``) gets the addition, an RMS norm and the convolution in one
    launch when every entry brings one token; for portions one launch adds and leaves every row's scale, and the
    convolution reads the stream itself, so the normed rows are never written.  Padding is told by its missing place in
    the mixer's cache, where it keeps one.

    params: hidden_size, taps, mixer (a PartSpec)."""

    graph_safe = True
    tape_safe = True

    @staticmethod
    def weight_specs(spec: PartSpec) -> Dict[str, WeightSpec]:
        sub: PartSpec = spec.params["mixer"]
        w = {f"mixer.{name}": ws for name, ws in MIXERS.get(sub.kind).weight_specs(sub).items()}
        w["taps"] = WeightSpec((int(spec.params["hidden_size"]), int(spec.params["taps"])))
        return w

    def __init__(self, spec: PartSpec, weights: Dict[str, torch.Tensor], rt: Runtime):
        super().__init__(spec, weights, rt)
        self.hidden, self.taps = int(spec.params["hidden_size"]), int(spec.params["taps"])
        if not (1 <= self.taps <= ops.sublayers.CONV_MAX_TAPS):
            raise ValueError(f"input_convolution: taps must lie in 1..{ops.sublayers.CONV_MAX_TAPS}")
        sub: PartSpec = spec.params["mixer"]
        local = {k[len("mixer."):]: t for k, t in weights.items() if k.startswith("mixer.")}
        self.mixer = MIXERS.get(sub.kind)(sub, local, rt)
        for p in vars(self.mixer).values():      # a mixer's position encoding is a part of its own for whoever walks the parts
            if isinstance(p, Part):
                self.position = p
        self.conv_w = weights["taps"].float().t().contiguous()      # [taps, hidden]: a tap's row is read as a row of h is
        inner = self.mixer.state_request()
        if inner is not None and (len(inner.shape) != 1 or inner.dtype != torch.float32):
            raise ValueError("input_convolution: the mixer's state must be one float32 row")
        self.inner_floats = int(inner.shape[0]) if inner is not None else 0
        self.tail_at = -(-self.inner_floats // 4) * 4
        self.state_floats = -(-(self.tail_at + (self.taps - 1) * self.hidden) // 4) * 4
        self.padding_safe = bool(self.mixer.padding_safe) and self.mixer.cache_request() is not None
        self.graph_safe = bool(self.mixer.graph_safe)
        self.tape_safe = bool(self.mixer.tape_safe)

    # ---- what the mixer asks for, and the tail beside it --------------------------------------------------------------
    def planner(self):
        return self.mixer.planner()

    def cache_request(self) -> Optional[KVCacheRequest]:
        return self.mixer.cache_request()

    def side_cache_requests(self) -> Dict[str, KVCacheRequest]:
        return self.mixer.side_cache_requests()

    def state_request(self) -> Optional[StateRequest]:
        return StateRequest((self.state_floats,), torch.float32) if self.state_floats else None

    def step_rows(self, rows: int, kind: str) -> int:
        return self.mixer.step_rows(rows, kind)

    def tune(self, num_tokens: int) -> None:
        self.mixer.tune(num_tokens)

    # ---- one step -----------------------------------------------------------------------------------------------------
    def _parts_of(self, batch, memory: LayerMemory):
        """(the mixer's memory, the tails, the tokens' places in the mixer's cache or None)."""
        state = memory.state
        inner = replace(memory, state=state[:, :self.inner_floats] if self.inner_floats else None)
        tail = state[:, self.tail_at:self.tail_at + (self.taps - 1) * self.hidden] if self.taps > 1 else None
        return inner, tail, batch.groups[memory.group].slots if memory.group >= 0 else None

    def forward(self, x: torch.Tensor, batch, memory: LayerMemory) -> torch.Tensor:
        inner, tail, slots = self._parts_of(batch, memory)
        h = ops.input_conv(x, self.conv_w, tail, batch.tok_seq, batch.entry_start, batch.entry_len, batch.entry_slot,
                           out=self.rt.buffer("mixer_in", (x.shape[0], self.hidden)), slots=slots)
        return self.mixer.forward(h, batch, inner)

    def forward_from_stream(self, norm, resid: torch.Tensor, delta: Optional[torch.Tensor], batch,
                            memory: LayerMemory) -> torch.Tensor:
        """resid += delta, then the mixer on its norm: the block's first norm is made here, with the convolution."""
        if not isinstance(norm, RMSNorm):
            x = norm.add_forward(resid, delta) if delta is not None else norm.forward(resid)
            return self.forward(x, batch, memory)
        n, rt = resid.shape[0], self.rt
        inner, tail, slots = self._parts_of(batch, memory)
        gain, add = norm.weight, 1.0 if norm.add_one else 0.0
        h = rt.buffer("mixer_in", (n, self.hidden))
        if batch.single_tokens and ops.norm_input_conv_supported(self.hidden, self.taps, delta):
            ops.norm_input_conv(resid, delta, gain, add, norm.eps, self.conv_w, tail, batch.tok_seq, batch.entry_slot,
                                out=h, slots=slots)
        else:
            scale = ops.stream_scale(resid, delta, norm.eps, out=rt.buffer("stream_scale", (n,), torch.float32))
            ops.input_conv(resid, self.conv_w, tail, batch.tok_seq, batch.entry_start, batch.entry_len, batch.entry_slot,
                           out=h, scale=scale, gain=gain, gain_add=add, slots=slots)
        return self.mixer.forward(h, batch, inner)
