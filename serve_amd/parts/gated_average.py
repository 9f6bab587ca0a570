"""A recurrent mixer without matrices in its memory: per channel an average whose gate reads the current token alone
(the form known as minGRU):

    z = sigmoid(W_z h + b_z),  u = W_x h + b_x,  c = u + 1/2 where u >= 0, else sigmoid(u)
    S_t = (1 - z) S_(t-1) + z c,      out = W_o (S_t * silu(W_g h))

z, x, g: `width` x the model's size.  Per-request state: S, one fp32 row (zero at admission).  Gates, candidates and the
recurrence are fp32 in both engines; the projections of z, x and g are one product with fp32 results.
"""
from __future__ import annotations

from typing import List

import torch

from .. import ops
from ..registry import register_part
from .base import LayerCache, ParamRequest, Part, Runtime, StateRequest
from .linear import linear
from .standard import _prepare_products


class GatedAverageMixer(Part):
    graph_safe = True

    def __init__(self, hidden_size: int, width: int):
        if width <= 0:
            raise ValueError("the width must be positive")
        self.hidden_size, self.width = int(hidden_size), int(width)

    def param_requests(self) -> List[ParamRequest]:
        d, W = self.hidden_size, self.width
        return [ParamRequest("z", (W, d), init="normal:0.08"), ParamRequest("z.b", (W,), init="normal:1.0"),
                ParamRequest("x", (W, d), init="normal:0.08"), ParamRequest("x.b", (W,), init="normal:0.3"),
                ParamRequest("g", (W, d), init="normal:0.08"), ParamRequest("o", (d, W), init="normal:0.08")]

    def state_request(self) -> StateRequest:
        return StateRequest((self.width,), torch.float32)

    def load(self, tensors, rt: Runtime) -> None:
        self.rt = rt
        big = [tensors[n] for n in ("z", "x", "g")]
        dt = big[0].dtype if all(t.dtype == big[0].dtype for t in big) else torch.float32
        self.w_in = torch.cat([t.to(dt) for t in big], dim=0).contiguous()        # one product: z | x | g
        self.b_in = torch.cat([tensors["z.b"].float(), tensors["x.b"].float()]).contiguous()
        self.wo = tensors["o"]
        _prepare_products(rt, self.w_in)

    def forward(self, h: torch.Tensor, ctx, cache: LayerCache, writes_cache: bool = True) -> torch.Tensor:
        if cache.state is None:
            raise ValueError("the gated average needs its per-request state")
        zxg = linear(h, self.w_in, out_dtype=torch.float32, partial_ok=True)       # (partial sums: the kernel adds them)
        y = ops.gated_average(zxg, self.b_in, cache.state, ctx, self.rt.empty((h.shape[0], self.width)))
        return linear(y, self.wo, partial_ok=True)


register_part("mixer", "gated_average", GatedAverageMixer)
