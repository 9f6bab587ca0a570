"""A residual stream of S copies (hyper-connections): x is fp32 [T, S, d], and every sublayer f of a layer (its mixer, its
feed-forward) reads a weighted sum of the copies and writes back to all of them,

    u = sum_s a_s x_s;   y = f(N(u) w);   x_t <- sum_s M_st x_s + b_t y            (all copies at once from the old ones)

with the sublayer's own `in` (a), `mix` (M, indexed [from, to]) and `out` (b).

`HyperResidual` (an arrangement) folds every update into the kernel that makes the next sublayer's input: what a sublayer
left, the matrix it goes through and the norm that follows are one kernel (`ops.stream_mix`), also from one layer to the
next, where they travel as a `StreamUpdate`, and into the final norm (`merged_streams_rmsnorm`: the sum of the copies).
Experts' rows are added up there as well, and the bias of a mixer's output joins it there.
The embedding starts equal copies (`token_embedding` with `copies`)."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, List, Optional

import torch

from .. import ops
from ..registry import register_part
from .base import LayerCache, ParamRequest, Part, Runtime, StepCost
from .standard import RMSNorm


class StreamWeights(Part):
    """One sublayer's weights on the copies."""

    graph_safe = True

    def __init__(self, streams: int):
        if not 0 < int(streams) <= ops.STREAM_MIX_MAX_STREAMS:
            raise ValueError(f"1 to {ops.STREAM_MIX_MAX_STREAMS} streams are taken, got {streams}")
        self.streams = int(streams)

    def param_requests(self) -> List[ParamRequest]:
        S = self.streams
        return [ParamRequest("in", (S,), init="uniform:0.1:0.6"), ParamRequest("out", (S,), init="ones_normal:0.3"),
                ParamRequest("mix", (S, S), init="uniform:0.05:0.45")]

    def step_cost(self, tokens: int, context_before: int = 0) -> StepCost:
        """The copies are mixed on the vector units beside a pass over memory: counted as weights, not as a product."""
        return StepCost(self.streams * (self.streams + 2), 0.0)

    def load(self, tensors, rt: Runtime) -> None:
        self.rt = rt
        self.from_ = tensors["in"].float().contiguous()
        self.to = tensors["out"].float().contiguous()
        self.mix = tensors["mix"].float().contiguous()


@dataclass
class StreamUpdate:
    """A sublayer's output on its way into the copies: y as `ops.stream_mix` takes it, a bias of it, its weights."""

    y: object
    bias: Optional[torch.Tensor]
    weights: StreamWeights


def _mix(x: torch.Tensor, pending: Optional[StreamUpdate], from_: torch.Tensor, norm: "RMSNorm", rt: Runtime,
         rows: Optional[torch.Tensor] = None) -> torch.Tensor:
    """Apply `pending` to the copies and return the norm of their sum with the weights `from_`."""
    if x.dim() != 3 or x.shape[1] != from_.numel():
        raise ValueError(f"the stream holds {list(x.shape[1:])}, {from_.numel()} copies are needed")
    if pending is not None and not isinstance(pending, StreamUpdate):
        raise ValueError("a stream of several copies is left by a layer that knows them")
    out = rt.empty((x.shape[0] if rows is None else rows.numel(), x.shape[2]))
    if pending is None:
        return ops.stream_mix(x, None, None, None, None, from_, norm.weight_f32, norm.eps, out, rows)
    p = pending
    return ops.stream_mix(x, p.y, p.bias, p.weights.mix, p.weights.to, from_, norm.weight_f32, norm.eps, out, rows)


class HyperResidual:
    """The arrangement: mixer and (optional) feed-forward, a norm and stream weights for each.  What it returns is the last
    sublayer's update, for the layer or the final norm behind it."""

    PART_ROLES = {"mixer": "mixer", "ffn": "feed_forward", "mixer_norm": "norm", "ffn_norm": "norm",
                  "mixer_streams": "stream_weights", "ffn_streams": "stream_weights"}
    OPTIONAL_PARTS = ("ffn", "ffn_norm", "ffn_streams")
    adds_output_bias = True

    def __init__(self, mixer, mixer_norm, mixer_streams, ffn=None, ffn_norm=None, ffn_streams=None):
        if not ((ffn is None) == (ffn_norm is None) == (ffn_streams is None)):
            raise ValueError("a feed-forward, its norm and its stream weights come together")
        self.mixer, self.mixer_norm, self.mixer_streams = mixer, mixer_norm, mixer_streams
        self.ffn, self.ffn_norm, self.ffn_streams = ffn, ffn_norm, ffn_streams

    def cache_owner(self) -> Part:
        return self.mixer

    def parts(self) -> Dict[str, Part]:
        out = {"mixer": self.mixer, "mixer_norm": self.mixer_norm, "mixer_streams": self.mixer_streams}
        if self.ffn is not None:
            out.update(ffn=self.ffn, ffn_norm=self.ffn_norm, ffn_streams=self.ffn_streams)
        return out

    def forward(self, x: torch.Tensor, pending: Optional[StreamUpdate], ctx, cache: LayerCache,
                writes_cache: bool = True) -> StreamUpdate:
        rt = self.mixer_norm.rt
        h = _mix(x, pending, self.mixer_streams.from_, self.mixer_norm, rt)
        y = self.mixer.forward(h, ctx, cache, writes_cache)
        update = StreamUpdate(y, getattr(self.mixer, "output_bias", None), self.mixer_streams)
        if self.ffn is None:
            return update
        h = _mix(x, update, self.ffn_streams.from_, self.ffn_norm, rt)
        if getattr(self.ffn, "leaves_rows", False):
            y = self.ffn.forward(h, ctx, rows_ok=True)          # (the next stream kernel adds the experts' rows up)
        else:
            y = self.ffn.forward(h, ctx)
        return StreamUpdate(y, getattr(self.ffn, "output_bias", None), self.ffn_streams)


class MergedStreamsNorm(RMSNorm):
    """The norm behind the last layer: of the sum of the copies, the last update included."""

    def __init__(self, size: int, eps: float, streams: int):
        super().__init__(size, eps)
        self.streams = int(streams)

    def load(self, tensors, rt: Runtime) -> None:
        super().load(tensors, rt)
        self.ones = torch.ones(self.streams, dtype=torch.float32, device=rt.device)

    def forward(self, x: torch.Tensor, delta, rows: Optional[torch.Tensor] = None, after=None) -> torch.Tensor:
        if after is not None:
            raise ValueError("nothing joins a stream of several copies behind this norm")
        return _mix(x, delta, self.ones, self, self.rt, rows)


register_part("stream_weights", "hyper_connection", StreamWeights)
register_part("arrangement", "hyper_residual", HyperResidual)
register_part("norm", "merged_streams_rmsnorm", MergedStreamsNorm)
