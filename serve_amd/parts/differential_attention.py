"""Differential attention: every head is two attentions (maps) over the same values, and the second is taken off the first:

    q, k (2 maps of `dim` per head), v = W h + b, each channel then through a short causal convolution over time
    q, k <- the first rot dims of every map turned by the position
    a_m  = softmax_j(scale q_m . k_m) v          over the keys j <= i, m = 1, 2
    o    = N(a_1 - lambda a_2) (1 - diff) * sigmoid(W_g h),   lambda = exp(lq1 . lk1) - exp(lq2 . lk2) + diff
    out  = W_o [o_1 .. o_H] + b_o                N(y) = y / sqrt(mean(y^2) + eps) over the head's values

The cache holds one key/value head per group: the maps' keys side by side and the values once.  Every (head, map) is a
query head with zeros outside its map, so that the paged attention kernels run unchanged (csrc/conv_attention.hip).

`conv`: the convolution's taps (the last on the current token; 0: none, and no `*.conv` tensors).  `bias`: biases of the
projections and of the output.  `own_kv=False`: the layer has no keys and values of its own and reads another layer's
(the run order says whose); its state is then its queries' alone.
Per-request state: the convolution's last taps - 1 inputs, one fp32 row.
"""
from __future__ import annotations

import math
from typing import List, Optional

import torch

from .. import ops, trace
from ..config.spec import PartSpec
from ..registry import get_part, register_part
from .base import LayerCache, ParamRequest, Part, Runtime, StateRequest, StepCost, TokenCacheRequest, keys_seen, kv_cache_request
from .linear import linear
from .normed_attention import padded_head_size
from .standard import _prepare_products

MAPS = 2


class DifferentialAttention(Part):
    graph_safe = True

    def __init__(self, hidden_size: int, num_heads: int, num_kv_heads: int, dim: int, vdim: int, scale: float, eps: float,
                 diff: float, position: Optional[PartSpec] = None, conv: int = 0, bias: bool = True, out_gate: bool = True,
                 own_kv: bool = True):
        if num_heads % num_kv_heads:
            raise ValueError("num_heads must be a multiple of num_kv_heads")
        if not 0 <= conv <= ops.CONV_ATTENTION_MAX_TAPS:
            raise ValueError(f"up to {ops.CONV_ATTENTION_MAX_TAPS} taps are taken, got {conv}")
        self.hidden_size, self.num_heads, self.num_kv_heads = int(hidden_size), int(num_heads), int(num_kv_heads)
        self.dim, self.vdim, self.scale, self.eps = int(dim), int(vdim), float(scale), float(eps)
        self.diff, self.taps, self.bias = float(diff), int(conv), bool(bias)
        self.out_gate, self.own_kv = bool(out_gate), bool(own_kv)
        self.has_output_bias = self.bias
        self.head_size = padded_head_size(MAPS * self.dim, self.vdim)
        if self.head_size > ops.SIMPLE_ATTENTION_MAX_HEAD_DIM:
            raise ValueError(f"twice dim and vdim may be up to {ops.SIMPLE_ATTENTION_MAX_HEAD_DIM}, got {self.head_size}")
        self.channels = MAPS * self.num_heads * self.dim                       # what the convolution sees
        if self.own_kv:
            self.channels += self.num_kv_heads * (MAPS * self.dim + self.vdim)
        self.position = None
        if position is not None:
            if not isinstance(position, PartSpec):
                position = PartSpec(position["kind"], position["params"])
            self.position = get_part("position", position.kind)(**position.params)
            self.graph_safe = bool(getattr(self.position, "graph_safe", False))

    def _projections(self):
        out = {"q": MAPS * self.num_heads * self.dim}
        if self.own_kv:
            out.update(k=MAPS * self.num_kv_heads * self.dim, v=self.num_kv_heads * self.vdim)
        return out

    def param_requests(self) -> List[ParamRequest]:
        d, H, Dv = self.hidden_size, self.num_heads, self.vdim
        out = []
        for name, n in self._projections().items():
            out.append(ParamRequest(name, (n, d), init="normal:0.08"))
            if self.bias:
                out.append(ParamRequest(name + ".b", (n,), init="normal:0.3"))
            if self.taps:
                out.append(ParamRequest(name + ".conv", (n, self.taps), init="normal:0.5"))
        out += [ParamRequest(n, (self.dim,), init="normal:0.15") for n in ("lq1", "lk1", "lq2", "lk2")]
        if self.out_gate:
            out.append(ParamRequest("g", (H * Dv, d), init="normal:0.08"))
        out.append(ParamRequest("o", (d, H * Dv), init="normal:0.08"))
        if self.bias:
            out.append(ParamRequest("o.b", (d,), init="normal:0.3"))
        return out

    def cache_request(self) -> Optional[TokenCacheRequest]:
        return kv_cache_request(self.num_kv_heads, self.head_size) if self.own_kv else None

    def state_request(self) -> Optional[StateRequest]:
        if self.taps < 2:
            return None
        return StateRequest(((self.taps - 1) * self.channels,), torch.float32)

    def step_cost(self, tokens: int, context_before: int = 0) -> StepCost:
        """The projections, and per map scores (dim) and weighted values (vdim) over the keys each token sees."""
        cost = super().step_cost(tokens, context_before)
        cost.flops += 2.0 * MAPS * self.num_heads * (self.dim + self.vdim) * keys_seen(tokens, context_before)
        return cost

    def load(self, tensors, rt: Runtime) -> None:
        self.rt = rt
        names = list(self._projections())
        big = [tensors[n] for n in names] + ([tensors["g"]] if self.out_gate else [])
        dt = big[0].dtype if all(t.dtype == big[0].dtype for t in big) else torch.float32
        self.w_in = torch.cat([t.to(dt) for t in big], dim=0).contiguous()       # one product: q | k | v | gate
        self.b_in = torch.cat([tensors[n + ".b"].float() for n in names]).contiguous() if self.bias else None
        if self.taps:
            self.conv_w = torch.cat([tensors[n + ".conv"].float() for n in names], dim=0).contiguous()
        else:
            self.conv_w = torch.ones((self.channels, 1), dtype=torch.float32, device=rt.device)
        self.output_bias = tensors["o.b"].float().contiguous() if self.bias else None
        l = {n: tensors[n].double() for n in ("lq1", "lk1", "lq2", "lk2")}
        self.lam = math.exp(float((l["lq1"] * l["lk1"]).sum())) - math.exp(float((l["lq2"] * l["lk2"]).sum())) + self.diff
        self.wo = tensors["o"]
        self.inv_freq, self.rot_dim, self.adjacent = None, 0, False
        if self.position is not None:
            self.position.load({}, rt)
            rot = self.position.rotary()
            if rot is None or rot.magnitude != 1.0:
                raise ValueError("this attention takes a rotation without a magnitude, or no position part")
            self.inv_freq, self.rot_dim, self.adjacent = rot.inv_freq.contiguous(), int(rot.rot_dim), bool(rot.adjacent_pairs)
            if self.rot_dim > self.dim:
                raise ValueError(f"a rotation of {self.rot_dim} dims does not fit maps of {self.dim}")
        _prepare_products(rt, self.w_in)

    def forward(self, h: torch.Tensor, ctx, cache: LayerCache, writes_cache: bool = True) -> torch.Tensor:
        H, G, D, Dv, Dp = self.num_heads, self.num_kv_heads, self.dim, self.vdim, self.head_size
        T = h.shape[0]
        if writes_cache != self.own_kv:
            raise ValueError("this attention writes its own keys and values, or it has none and reads another layer's")
        if self.taps > 1 and cache.state is None:
            raise ValueError("the convolution needs its per-request state")
        if cache.k_pages.shape[-1] != Dp or cache.k_pages.shape[1] != G:
            raise ValueError(f"the cache keeps {cache.k_pages.shape[1]} heads of {cache.k_pages.shape[-1]}, this layer reads {G} of {Dp}")
        grp = ctx.groups[cache.group]
        with trace.span("write_to_cache"):
            z = linear(h, self.w_in)
            q = self.rt.empty((T, H * MAPS * Dp))
            ops.conv_rope_kv_write(z, self.b_in, self.conv_w, cache.state, 0, ctx, q, grp.slots if self.own_kv else None,
                                   cache.k_pages, cache.v_pages, self.inv_freq, self.rot_dim, self.adjacent, H, G, MAPS, D, Dv)
        attn = self.rt.empty((T, H * MAPS * Dp))
        with trace.span("attention"):
            ops.paged_attention(q, H * MAPS * Dp, attn, cache.k_pages, cache.v_pages, grp.block_table, ctx, H * MAPS,
                                self.scale, None)
        y = self.rt.empty((T, H * Dv))
        ops.differential_heads(attn, z if self.out_gate else None, self.channels, y, self.lam, 1.0 - self.diff, self.eps, H, Dv)
        return linear(y, self.wo, partial_ok=True)      # the consumer adds the parts


register_part("mixer", "differential_attention", DifferentialAttention)
