"""Several residual streams a token, and how a sublayer reads them and writes its result back."""
from __future__ import annotations

from typing import Dict, Optional, Tuple

import torch

from .. import ops
from ..config.forward_config import PartSpec
from ..weights.loader import WeightSpec
from .base import Part, Runtime, register_connection

# a sublayer's result that has not been written into the streams yet, and the connection that writes it
Pending = Optional[Tuple["HyperConnection", torch.Tensor]]


class Streams:
    """The float32 residual streams of one step, [count, n, H].  Until the first result is written they are all equal to the
    embedding's output [n, H], which then stands for them.  A result stays pending until the next row is read: writing it,
    reading the next sublayer's row and norming that row are one launch (``ops.stream_mix``)."""

    def __init__(self, rt: Runtime, embedded: torch.Tensor, count: int):
        self.rt, self.count = rt, int(count)
        self.n, self.hidden = int(embedded.shape[0]), int(embedded.shape[1])
        self.values = embedded      # [n, H] (all streams equal) or [count, n, H]

    def _mix(self, pending: Pending, read: torch.Tensor, row_norm, name: str, keep: bool, rows=None) -> torch.Tensor:
        gain, eps, centered = row_norm
        m = self.n if rows is None else int(rows.numel())
        out = self.rt.buffer(name, (m, self.hidden))
        kw = {}
        if pending is not None:
            connection, y = pending
            kw = {"y": y, "write": connection.write, "scale": connection.scale}
            if keep:
                kw["keep"] = self.rt.buffer("streams", (self.count, self.n, self.hidden), torch.float32)
        ops.stream_mix(self.values, read, gain, eps, centered, out=out, rows=rows, **kw)
        if "keep" in kw:
            self.values = kw["keep"]
        return out

    def read(self, pending: Pending, connection: "HyperConnection", row_norm) -> torch.Tensor:
        """The pending result is written; what ``connection`` reads comes back normed, in the activation type."""
        return self._mix(pending, connection.read_weights, row_norm, "norm_out", keep=True)

    def finish(self, pending: Pending, ones: torch.Tensor, row_norm, rows=None) -> torch.Tensor:
        """The sum of the streams (with the pending result in it), normed; of the rows ``rows`` alone if given.  The streams
        themselves are left as they are."""
        return self._mix(pending, ones, row_norm, "norm_out" if rows is None else "norm_rows", keep=False, rows=rows)


@register_connection("hyper")
class HyperConnection(Part):
    """The row a sublayer reads is sum_s in[s] X_s; its result y changes all streams at once, from the old ones:
    X_t <- sum_s mix[s, t] X_s + mult * out[t] * (y * scale).

    params: streams, hidden_size, mult (1), scale (False: no gains on y).
    weights: in, out [streams], mix [streams, streams] (from, to), scale [hidden_size]."""

    graph_safe = True
    tape_safe = True

    @staticmethod
    def weight_specs(spec: PartSpec) -> Dict[str, WeightSpec]:
        s = int(spec.params["streams"])
        w = {"in": WeightSpec((s,), init="ones"), "out": WeightSpec((s,), init="ones"), "mix": WeightSpec((s, s), init="eye")}
        if spec.params.get("scale", False):
            w["scale"] = WeightSpec((int(spec.params["hidden_size"]),), init="ones")
        return w

    def __init__(self, spec: PartSpec, weights: Dict[str, torch.Tensor], rt: Runtime):
        super().__init__(spec, weights, rt)
        mult = float(spec.params.get("mult", 1.0))
        self.read_weights = weights["in"].float().contiguous()
        self.write = torch.cat([weights["mix"].float().reshape(-1), weights["out"].float() * mult]).contiguous()
        self.scale = weights["scale"].float().contiguous() if spec.params.get("scale", False) else None


@register_connection("none")
class NoConnection(Part):
    """Stands where an arrangement names the connection of a sublayer that a layer does not have."""

    graph_safe = True
    tape_safe = True
