"""The parts of the dense Llama decoder: RMSNorm, rotary position encoding, grouped-query
attention over the paged cache, SwiGLU feed-forward, token embedding, output head, and the
pre-norm residual arrangement of a layer.  Each takes its sizes and constants as parameters.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch

from .. import ops, trace
from ..config.spec import PartSpec
from ..registry import get_part, register_part
from .base import (NORMED_STREAM, LayerCache, ParamRequest, Part, PositionPart, Rotary, Runtime, StepCost, TokenCacheRequest,
                   kv_cache_request)
from .linear import linear


def _prepare_products(rt: Runtime, weight: torch.Tensor) -> None:
    """What the products over `weight` need beside their operands, made when a part loads and not
    at its first step (which may run inside a graph capture): the library's scratch memory."""
    if weight.is_cuda and weight.dtype == torch.bfloat16 and rt.dtype == torch.bfloat16:
        ops.blaslt_workspace(weight.device)


# ---------------------------------------------------------------------------------------------
# norm
# ---------------------------------------------------------------------------------------------
class RMSNorm(Part):
    """y = x * rsqrt(mean(x^2) + eps) * weight (serve/model.py:57-68), fused with the addition
    of the previous part's output into the fp32 residual stream (serve/model.py:147-148)."""

    graph_safe = True

    def __init__(self, size: int, eps: float, offset: float = 0.0):
        """`offset`: what is added to the stored weight before it multiplies (1.0 for checkpoints
        that keep their norm weights around zero); the sum is made in fp32 when the part loads."""
        self.size, self.eps, self.offset = int(size), float(eps), float(offset)

    def param_requests(self) -> List[ParamRequest]:
        return [ParamRequest("weight", (self.size,), init="normal:0.2" if self.offset else "ones_normal")]

    def load(self, tensors, rt: Runtime) -> None:
        self.rt = rt
        self.weight = tensors["weight"]
        if self.offset:
            self.weight = self.weight.float() + self.offset
        # (for kernels that apply this norm at the end of another kernel's work and take fp32 vectors)
        self.weight_f32 = self.weight if self.weight.dtype == torch.float32 else self.weight.float()

    def forward(self, x: torch.Tensor, delta: Optional[torch.Tensor], rows: Optional[torch.Tensor] = None,
                after: Optional[torch.Tensor] = None) -> torch.Tensor:
        n = x.shape[0] if rows is None else rows.numel()
        out = self.rt.empty((n, self.size))
        return ops.add_rmsnorm(x, delta, self.weight, self.eps, out, rows, after)


# ---------------------------------------------------------------------------------------------
# position encoding
# ---------------------------------------------------------------------------------------------
def rope_inverse_frequencies(head_dim_rot: int, theta: float, scaling: Optional[dict]) -> torch.Tensor:
    """f_j = theta^(-2j/rot), j < rot/2, in fp32 (serve/model.py:276), then the llama3 rescale of
    serve/model.py:247-266: wavelengths below orig/high_freq_factor keep f, above
    orig/low_freq_factor get f/factor, between them the two are blended linearly in
    orig/wavelength."""
    f = 1.0 / (theta ** (torch.arange(0, head_dim_rot, 2, dtype=torch.int64)[: head_dim_rot // 2].float()
                         / head_dim_rot))
    if scaling is None:
        return f
    kind = scaling.get("rope_type", scaling.get("type", "llama3"))
    if kind == "yarn":
        return yarn_frequencies(head_dim_rot, theta, scaling)[0]
    if kind == "linear":
        # every frequency divided by the factor; float64, rounded once
        if not float(scaling["factor"]) > 0:
            raise ValueError("linear scaling needs a positive factor")
        i = torch.arange(head_dim_rot // 2, dtype=torch.float64)
        return (float(theta) ** (-2.0 * i / head_dim_rot) / float(scaling["factor"])).float()
    if kind != "llama3":
        raise ValueError(f"rope scaling {kind!r} is not supported (known: 'llama3', 'yarn', 'linear')")
    factor = float(scaling["factor"])
    low = float(scaling["low_freq_factor"])
    high = float(scaling["high_freq_factor"])
    orig = float(scaling["original_max_position_embeddings"])
    wavelen = 2 * math.pi / f
    smooth = (orig / wavelen - low) / (high - low)
    blended = (1 - smooth) * f / factor + smooth * f
    out = torch.where(wavelen < orig / high, f, torch.where(wavelen > orig / low, f / factor, blended))
    return out.float()


def yarn_frequencies(rot_dim: int, theta: float, scaling: dict):
    """(frequencies fp32 [rot_dim / 2], magnitude) of a rotation stretched to longer contexts by blending, per
    pair, the plain frequency f_i = theta^(-2i/rot_dim) with f_i / factor:

        turns(n) = rot_dim ln(original / (2 pi n)) / (2 ln theta)      the pair that makes n turns over `original` positions
        lo = max(floor(turns(fast)), 0),  hi = min(ceil(turns(slow)), rot_dim - 1)
        ramp_i = clamp((i - lo) / max(hi - lo, 0.001), 0, 1)
        f_i' = f_i / factor * ramp_i + f_i (1 - ramp_i)

    and sine and cosine are multiplied by 0.1 ln(factor) + 1.  Keys of `scaling`: factor, original, fast, slow.
    Computed in float64 and rounded once."""
    factor, original = float(scaling["factor"]), float(scaling["original"])
    fast, slow = float(scaling["fast"]), float(scaling["slow"])
    if not (factor > 0 and original > 0 and fast > 0 and slow > 0 and theta > 1):
        raise ValueError("yarn scaling needs positive factor, original, fast and slow, and a base above 1")
    i = torch.arange(rot_dim // 2, dtype=torch.float64)
    f = float(theta) ** (-2.0 * i / rot_dim)

    def turns(n: float) -> float:
        return rot_dim * math.log(original / (2.0 * math.pi * n)) / (2.0 * math.log(theta))

    lo = max(math.floor(turns(fast)), 0)
    hi = min(math.ceil(turns(slow)), rot_dim - 1)
    ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0.0, 1.0)
    return (f / factor * ramp + f * (1.0 - ramp)).float(), 0.1 * math.log(factor) + 1.0


# largest angle (position * frequency, in radians) whose sine and cosine the bfloat16 kernels'
# own argument reduction gives to 1e-6; the float32 kernels use the library's sincosf
ROTARY_MAX_ANGLE_REDUCED = 4.0e6


class RotaryPosition(PositionPart):
    """Rotation of pairs of q and k by position * f_j (serve/model.py:234-244).

    `pairing="half"`: pair j is (j, j + rot/2), the row order of checkpoints; the reference
    reaches the same scores by permuting the q/k rows and rotating adjacent pairs
    (serve/hf_utils/convert_hf_checkpoint.py:115-118), which is `pairing="adjacent"`.
    `rot_dim < head_dim` leaves the remaining dims of every head as they are.  The part only
    says what the rotation is (`rotary()`); the attention's kernels carry it out, fused with
    the projection or the cache write.  `scaling` with `rope_type` "llama3", "yarn" or "linear" (see
    `rope_inverse_frequencies`, `yarn_frequencies`); "yarn" also gives the rotation a magnitude."""

    graph_safe = True

    def __init__(self, head_dim: int, rot_dim: int, theta: float, scaling: Optional[dict] = None,
                 pairing: str = "half"):
        if pairing not in ("half", "adjacent"):
            raise ValueError(f"pairing must be 'half' or 'adjacent', got {pairing!r}")
        if rot_dim % 2 or not 0 < rot_dim <= head_dim:
            raise ValueError(f"rot_dim {rot_dim} must be even and within head_dim {head_dim}")
        self.head_dim, self.rot_dim = int(head_dim), int(rot_dim)
        self.theta, self.scaling, self.pairing = float(theta), scaling, pairing

    def load(self, tensors, rt: Runtime) -> None:
        self.rt = rt
        f = rope_inverse_frequencies(self.rot_dim, self.theta, self.scaling)
        if not rt.exact and rt.max_context is not None:
            top = float(f.max()) * max(rt.max_context - 1, 0)
            if top > ROTARY_MAX_ANGLE_REDUCED:
                raise ValueError(f"a context of {rt.max_context} tokens gives rotation angles up to {top:.3g} rad; "
                                 f"the bfloat16 kernels hold up to {ROTARY_MAX_ANGLE_REDUCED:.3g} "
                                 "(use dtype float32, or a shorter max_context)")
        magnitude = 1.0
        if self.scaling is not None and self.scaling.get("rope_type", self.scaling.get("type")) == "yarn":
            magnitude = yarn_frequencies(self.rot_dim, self.theta, self.scaling)[1]
        self._rotary = Rotary(f.to(rt.device), self.rot_dim, self.pairing == "adjacent", magnitude)

    def rotary(self) -> Rotary:
        return self._rotary


# ---------------------------------------------------------------------------------------------
# mixer: grouped-query attention
# ---------------------------------------------------------------------------------------------
class GQAAttention(Part):
    """q, k, v in one product, rotate q and k, store k and v in the paged cache, attend over the
    cache, project back (serve/model.py:88-134).  Query head h reads KV head h // (Hq // Hk)."""

    graph_safe = True

    def __init__(self, hidden_size: int, num_heads: int, num_kv_heads: int, head_dim: int, scale: float,
                 position: PartSpec, window: Optional[int] = None):
        if num_heads % num_kv_heads:
            raise ValueError("num_heads must be a multiple of num_kv_heads")
        self.hidden_size, self.num_heads, self.num_kv_heads = int(hidden_size), int(num_heads), int(num_kv_heads)
        self.head_dim, self.scale, self.window = int(head_dim), float(scale), window
        if not isinstance(position, PartSpec):
            position = PartSpec(position["kind"], position["params"])
        self.position = get_part("position", position.kind)(**position.params)
        # a position part that reads back to the host keeps the whole mixer out of graphs
        self.graph_safe = bool(getattr(self.position, "graph_safe", False))

    def param_requests(self) -> List[ParamRequest]:
        d, D = self.hidden_size, self.head_dim
        return [ParamRequest("q_proj.weight", (self.num_heads * D, d)),
                ParamRequest("k_proj.weight", (self.num_kv_heads * D, d)),
                ParamRequest("v_proj.weight", (self.num_kv_heads * D, d)),
                ParamRequest("o_proj.weight", (d, self.num_heads * D))]

    def cache_request(self) -> TokenCacheRequest:
        return kv_cache_request(self.num_kv_heads, self.head_dim, self.window)

    def step_cost(self, tokens: int, context_before: int = 0) -> StepCost:
        """The four projections, and scores and weighted values over the keys each token sees: token j
        of the portion sees context_before + j + 1 keys (at most `window`), two products of head_dim
        multiply-adds per key and query head."""
        cost = super().step_cost(tokens, context_before)
        if self.window:
            keys = sum(min(context_before + j + 1, self.window) for j in range(tokens))
        else:
            keys = tokens * context_before + tokens * (tokens + 1) // 2
        cost.flops += 4.0 * self.num_heads * self.head_dim * keys
        return cost

    def load(self, tensors, rt: Runtime) -> None:
        self.rt = rt
        parts = [tensors["q_proj.weight"], tensors["k_proj.weight"], tensors["v_proj.weight"]]
        dt = parts[0].dtype if all(p.dtype == parts[0].dtype for p in parts) else torch.float32
        # one product for q, k and v (serve/model.py:95,104-108)
        self.wqkv = torch.cat([p.to(dt) for p in parts], dim=0).contiguous()
        self.wq = self.wqkv[: self.num_heads * self.head_dim]
        self.wo = tensors["o_proj.weight"]
        _prepare_products(rt, self.wqkv)
        self.position.load({}, rt)
        rot = self.position.rotary()
        if rot is not None and rot.magnitude != 1.0:
            raise ValueError("this attention's kernels rotate without a magnitude; the kind 'rotary_attention' takes one")
        self._no_freq = torch.empty(0, dtype=torch.float32, device=rt.device)

    def _project_encode_store(self, h: torch.Tensor, ctx, cache: LayerCache, slots: Optional[torch.Tensor]):
        """q (with k and v behind it in the same rows when they are stored), encoded by position,
        k and v written to the token's cache slots.  Returns the rows: [T, Hq D] (q alone) or
        [T, (Hq + 2 Hk) D]; either way q is their first Hq D columns."""
        Hq, Hk, D = self.num_heads, self.num_kv_heads, self.head_dim
        store = slots is not None
        rot = self.position.rotary()
        if (store and rot is not None
                and ops.qkv_rope_available(h, self.wqkv, cache.k_pages, D, rot.rot_dim, rot.adjacent_pairs)):
            # few rows: product, rotation and cache write are one kernel; only q comes back
            q = self.rt.empty((h.shape[0], Hq * D))
            return ops.qkv_rope_bf16(h, self.wqkv, q, ctx.positions, rot.inv_freq, slots, cache.k_pages,
                                     cache.v_pages, Hq, Hk, D, cache.page_size)
        qkv = linear(h, self.wqkv if store else self.wq)
        if rot is None:
            # an encoding the kernels do not know: the position part works on q and k itself
            T = qkv.shape[0]
            k = qkv[:, Hq * D: (Hq + Hk) * D].view(T, Hk, D) if store else None
            self.position.apply(qkv[:, : Hq * D].view(T, Hq, D), k, ctx.positions)
            if not store:
                return qkv
            inv_freq, rot_dim, adjacent = self._no_freq, 0, False
        else:
            inv_freq, rot_dim, adjacent = rot.inv_freq, rot.rot_dim, rot.adjacent_pairs
        ops.rope_kv_write(qkv, ctx.positions, inv_freq, slots, cache.k_pages if store else None,
                          cache.v_pages if store else None, Hq, Hk, D, rot_dim, adjacent,
                          max(cache.page_size, 1))
        return qkv

    def forward(self, h: torch.Tensor, ctx, cache: LayerCache, writes_cache: bool = True) -> torch.Tensor:
        grp = ctx.groups[cache.group]
        with trace.span("write_to_cache"):                 # (with the projection and the rotation; serve/model.py:122)
            qkv = self._project_encode_store(h, ctx, cache, grp.slots if writes_cache else None)
        attn = self.rt.empty((h.shape[0], self.num_heads * self.head_dim))
        with trace.span("attention"):                      # serve/model.py:127
            ops.paged_attention(qkv, qkv.shape[1], attn, cache.k_pages, cache.v_pages, grp.block_table, ctx,
                                self.num_heads, self.scale, self.window)
        return linear(attn, self.wo, partial_ok=True)      # the following norm adds the parts


# ---------------------------------------------------------------------------------------------
# feed-forward
# ---------------------------------------------------------------------------------------------
class SwiGLU(Part):
    """down(silu(gate x) * up x), no biases (serve/model.py:71-85); gate and up run as one
    product over the stacked matrix.  `activation` names another gate of `ops.GATES` in place of
    silu(g) u: "gelu_tanh", or "clamped_swish" with its `limit`."""

    graph_safe = True

    def __init__(self, hidden_size: int, intermediate_size: int, activation: str = "silu", limit: float = 0.0):
        if activation not in ops.GATES:
            raise ValueError(f"unknown gate {activation!r}; known: {sorted(ops.GATES)}")
        if activation == "clamped_swish" and not limit > 0.0:
            raise ValueError("the clamped gate needs a positive limit")
        self.hidden_size, self.intermediate_size = int(hidden_size), int(intermediate_size)
        self.activation, self.limit = activation, float(limit)

    def param_requests(self) -> List[ParamRequest]:
        d, i = self.hidden_size, self.intermediate_size
        return [ParamRequest("gate_proj.weight", (i, d)), ParamRequest("up_proj.weight", (i, d)),
                ParamRequest("down_proj.weight", (d, i))]

    def load(self, tensors, rt: Runtime) -> None:
        self.rt = rt
        g, u = tensors["gate_proj.weight"], tensors["up_proj.weight"]
        dt = g.dtype if g.dtype == u.dtype else torch.float32
        self.w_gate_up = torch.cat([g.to(dt), u.to(dt)], dim=0).contiguous()
        self.w_down = tensors["down_proj.weight"]
        _prepare_products(rt, self.w_down)

    def forward(self, h: torch.Tensor, ctx) -> torch.Tensor:
        a = self.rt.empty((h.shape[0], self.intermediate_size))
        M = h.shape[0]
        if (h.dtype == torch.bfloat16 and self.w_gate_up.dtype == torch.bfloat16
                and self.hidden_size % 8 == 0
                and (M <= ops.SKINNY_MAX_ROWS or (M <= ops.WIDE_MAX_ROWS and ops.gemm_takes_wide(
                    M, self.intermediate_size, self.hidden_size, 1, swiglu=True)))):
            ops.swiglu_bf16(h, self.w_gate_up, a, self.activation, self.limit)          # product and gate in one kernel
        else:
            gu = linear(h, self.w_gate_up)
            ops.gate_mul(gu, a, self.activation, self.limit)
        return linear(a, self.w_down, partial_ok=True)     # the following norm adds the parts


# ---------------------------------------------------------------------------------------------
# embedding and output head
# ---------------------------------------------------------------------------------------------
class TokenEmbedding(Part):
    """x = table[token] (serve/model.py:157,220); the residual stream it starts is fp32."""

    graph_safe = True

    def __init__(self, vocab_size: int, hidden_size: int, scale: float = 1.0, side_width: int = 0,
                 copies: int = 0):
        """`scale` multiplies every row as it enters the stream (in fp32; the table itself, which an
        output head may share, stays as stored).  `side_width` > 0: the part also holds a second table
        `side` [vocab, side_width], a second row per token that parts of the layers read (they name it as
        `embedding.side`); nothing of it enters the stream here.  `copies` > 0: the stream is [T, copies, d], equal copies."""
        self.vocab_size, self.hidden_size, self.scale = int(vocab_size), int(hidden_size), float(scale)
        self.side_width, self.copies = int(side_width), int(copies)

    def param_requests(self) -> List[ParamRequest]:
        out = [ParamRequest("weight", (self.vocab_size, self.hidden_size))]
        if self.side_width:
            out.append(ParamRequest("side", (self.vocab_size, self.side_width), init="normal:1.0"))
        return out

    def load(self, tensors, rt: Runtime) -> None:
        self.rt = rt
        self.weight = tensors["weight"]
        self.side = tensors.get("side")

    def step_cost(self, tokens: int, context_before: int = 0) -> StepCost:
        """A gather of `tokens` rows: no product, and of the table only those rows are read (not
        counted: a measurement that prices a step by the tensors it streams leaves them out)."""
        return StepCost(0, 0.0)

    def forward(self, ctx) -> torch.Tensor:
        """The rows of the step's tokens.  `ctx.src_row` / `ctx.prev_tokens` (when set): rows whose
        token was sampled on the device by an earlier step and never reached the host."""
        T = ctx.token_ids.numel()
        x = self.rt.empty((T, self.copies, self.hidden_size) if self.copies else (T, self.hidden_size), torch.float32)
        return ops.embed(self.weight, ctx.token_ids, x, ctx.src_row, ctx.prev_tokens, self.scale)


class LinearHead(Part):
    """logits = h @ W^T in fp32 (serve/model.py:159,226-231).  `shares` names the tensor of another
    part that serves as W when the checkpoint has none of its own; a `tied` head never reads its
    own (serve/hf_utils/convert_hf_checkpoint.py:146-147).  It then receives that tensor itself:
    no second copy of the table exists."""

    graph_safe = True

    def __init__(self, vocab_size: int, hidden_size: int, tied: bool = False,
                 shares: Optional[str] = "embedding.weight", scale: float = 1.0, soft_cap: float = 0.0):
        """`scale` multiplies the products; `soft_cap` > 0 then keeps them within it: cap tanh(logit / cap)."""
        self.vocab_size, self.hidden_size, self.tied = int(vocab_size), int(hidden_size), bool(tied)
        self.scale, self.soft_cap = float(scale), float(soft_cap)
        if self.soft_cap < 0:
            raise ValueError("a soft cap is positive, or 0 for none")
        self.shares = shares
        if self.tied and not shares:
            raise ValueError("a tied head needs the name of the tensor it shares")

    def param_requests(self) -> List[ParamRequest]:
        return [ParamRequest("weight", (self.vocab_size, self.hidden_size), alias_of=self.shares,
                             alias_only=self.tied)]

    def load(self, tensors, rt: Runtime) -> None:
        self.rt = rt
        self.weight = tensors["weight"]
        _prepare_products(rt, self.weight)

    accepts_out = True

    def forward(self, h: torch.Tensor, out: Optional[torch.Tensor] = None) -> torch.Tensor:
        """fp32 logits [R, V]; into `out` where the caller brings the buffer."""
        if out is not None and (out.shape != (h.shape[0], self.vocab_size) or out.dtype != torch.float32
                                or not out.is_contiguous()):
            raise ValueError(f"the logits buffer must be contiguous fp32 [{h.shape[0]}, {self.vocab_size}]")
        y = linear(h, self.weight, out_dtype=torch.float32, out=out)
        if self.scale != 1.0 or self.soft_cap:
            ops.scale_soft_cap(y, self.scale, self.soft_cap)
        return y


# ---------------------------------------------------------------------------------------------
# arrangement of a layer
# ---------------------------------------------------------------------------------------------
class PreNormResidual:
    """x = x + mixer(norm1(x)); x = x + ffn(norm2(x)) (serve/model.py:146-149).

    The additions are folded into the following norm: `pending` is the output of the previous
    part that has not been added to the residual stream yet; the layer returns its own.

    A bias of the mixer's output is a constant row: the mixer's norm adds it to the stream behind itself, which is where
    the mixer's output joins it too.

    A layer may have no feed-forward (then it has no `ffn_norm` either), and it may end with a
    `token_input`: a part that adds something made from the step's tokens and the finished stream
    (`forward(x, pending, ctx) -> pending`: it folds the layer's last output into x itself).  Such a part may
    apply the norm that the next layer begins with (`ctx.next_input_norm`) at the end of its own last kernel and
    leave the activations on the step's context; a layer that finds them there, made with its norm, starts from them."""

    PART_ROLES = {"mixer": "mixer", "ffn": "feed_forward", "mixer_norm": "norm", "ffn_norm": "norm",
                  "token_input": "token_input"}
    OPTIONAL_PARTS = ("ffn", "ffn_norm", "token_input")
    adds_output_bias = True

    def __init__(self, mixer, mixer_norm, ffn=None, ffn_norm=None, token_input=None):
        if (ffn is None) != (ffn_norm is None):
            raise ValueError("a feed-forward and its norm come together")
        if any(getattr(p, "has_output_bias", False) for p in (ffn, token_input)):
            raise ValueError("this arrangement adds the mixer's output bias, and no other part's")
        self.mixer, self.ffn, self.mixer_norm, self.ffn_norm = mixer, ffn, mixer_norm, ffn_norm
        self.token_input = token_input

    def cache_owner(self) -> Part:
        return self.mixer

    def parts(self) -> Dict[str, Part]:
        out = {"mixer": self.mixer, "mixer_norm": self.mixer_norm}
        if self.ffn is not None:
            out.update(ffn=self.ffn, ffn_norm=self.ffn_norm)
        if self.token_input is not None:
            out["token_input"] = self.token_input
        return out

    def input_norm(self) -> Part:
        """The norm this layer begins with: the layer before may apply it at the end of its own last kernel."""
        return self.mixer_norm

    def forward(self, x: torch.Tensor, pending: Optional[torch.Tensor], ctx, cache: LayerCache,
                writes_cache: bool = True) -> Optional[torch.Tensor]:
        ready = ctx.shared.pop(NORMED_STREAM, None) if getattr(ctx, "shared", None) else None
        bias = getattr(self.mixer, "output_bias", None)
        if ready is not None and ready[1] is self.mixer_norm and pending is None:
            h = ready[0]                            # the layer before has made it, with this layer's norm
            if bias is not None:
                ops.stream_add(x, None, bias)
        elif bias is not None:
            h = self.mixer_norm.forward(x, pending, after=bias)
        else:
            h = self.mixer_norm.forward(x, pending)
        a = self.mixer.forward(h, ctx, cache, writes_cache)
        if self.ffn is not None:
            h = self.ffn_norm.forward(x, a)
            a = self.ffn.forward(h, ctx)
        if self.token_input is not None:
            a = self.token_input.forward(x, a, ctx)
        return a


register_part("norm", "rmsnorm", RMSNorm)
register_part("position", "rope", RotaryPosition)
register_part("mixer", "gqa_attention", GQAAttention)
register_part("feed_forward", "swiglu", SwiGLU)
register_part("feed_forward", "gated", SwiGLU)            # (the same part under the name of its general form)
register_part("embedding", "token_embedding", TokenEmbedding)
register_part("lm_head", "linear_head", LinearHead)
register_part("arrangement", "prenorm_residual", PreNormResidual)
