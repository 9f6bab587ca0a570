"""A plain, slow implementation of the Topapel decoder in float64: one function per mechanism, whole sequences
at a time, no cache.  It shares no code with the package; the tests compare the engine with it.

    x_0    = scale_e E[token]
    layer:   x <- x + mixer(N(x) (1 + w_1));  then, where the layer has a feed-forward,  x <- x + ff(N(x) (1 + w_2))
    y      = E (N(x) (1 + w_f)) scale_l,      logits = cap tanh(y / cap)

A model is a dict: {"config": the configuration as config.json holds it, "tensors": {name: float64 tensor}}.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch

F64 = torch.float64


def over_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def stream_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """The norm in front of every sublayer and of the output: its weight is stored around zero."""
    return over_rms(x, eps) * (1.0 + w)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def embedding(tokens: List[int], table: torch.Tensor, scale: float) -> torch.Tensor:
    return table[torch.tensor(tokens)] * scale


# -- softmax attention ---------------------------------------------------------------------------------
def rotary_frequencies(dims: int, base: float, scaling: Optional[dict]) -> torch.Tensor:
    f = base ** (-2.0 * torch.arange(dims // 2, dtype=F64) / dims)
    return f / float(scaling["factor"]) if scaling else f


def rotate(x: torch.Tensor, positions: torch.Tensor, f: torch.Tensor) -> torch.Tensor:
    """x [T, H, D]: dims i and i + n (n = len(f)) of every head turned by position * f_i, the dims behind 2 n as they are."""
    n = f.numel()
    a = positions.to(F64)[:, None] * f[None, :]
    cos, sin = torch.cos(a)[:, None, :], torch.sin(a)[:, None, :]
    u, v = x[..., :n], x[..., n:2 * n]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, x[..., 2 * n:]], -1)


def seen_keys(T: int, chunk: Optional[int]) -> torch.Tensor:
    """[T, T] of bool: query i sees key j, j <= i and (with chunks) both in the same run of `chunk` positions."""
    i = torch.arange(T)
    seen = i[None, :] <= i[:, None]
    if chunk:
        seen &= (i // chunk)[None, :] == (i // chunk)[:, None]
    return seen


def sink_softmax(scores: torch.Tensor, seen: torch.Tensor, sink: torch.Tensor) -> torch.Tensor:
    """Rows of weights over the seen keys; the denominator has one more term exp(sink)."""
    s = scores.masked_fill(~seen, -math.inf)
    m = torch.maximum(s.max(-1, keepdim=True).values, sink)
    e = torch.exp(s - m)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink - m))


def attention_mixer(h: torch.Tensor, t: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    q = (h @ t[p + "q"].T + t[p + "q.b"]).view(T, H, D)
    k = (h @ t[p + "k"].T + t[p + "k.b"]).view(T, G, D)
    v = k                                                    # the values: the keys as they were projected
    q, k = over_rms(q, eps) * t[p + "q.norm"], over_rms(k, eps) * t[p + "k.norm"]
    rot = m.get("rot")
    if rot:
        f = rotary_frequencies(rot["dims"], rot["base"], rot.get("scaling"))
        q, k = rotate(q, torch.arange(T), f), rotate(k, torch.arange(T), f)
    seen = seen_keys(T, (m.get("mask") or {}).get("size"))
    out = torch.zeros((T, H, D), dtype=F64)
    for i in range(H):
        g = i // (H // G)
        w = sink_softmax(q[:, i] @ k[:, g].T * m["scale"], seen, t[p + "sink"][i])
        out[:, i] = w @ v[:, g]
    return out.reshape(T, H * D) @ t[p + "o"].T + t[p + "o.b"]


# -- recurrent mixers ----------------------------------------------------------------------------------
def decayed_outer_products(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay: torch.Tensor) -> torch.Tensor:
    """q, k [T, H, D], v [T, H, Dv], decay [H]: S <- decay S + k v^T per head, o = S^T q; [T, H, Dv]."""
    T, H, D = q.shape
    S = torch.zeros((H, D, v.shape[2]), dtype=F64)
    out = torch.zeros_like(v)
    for i in range(T):
        S = decay[:, None, None] * S + k[i][:, :, None] * v[i][:, None, :]
        out[i] = (S * q[i][:, :, None]).sum(1)
    return out


def lightning_mixer(h: torch.Tensor, t: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, D, Dv = m["heads"], m["dim"], m["vdim"]
    q, k = silu(h @ t[p + "q"].T).view(T, H, D), silu(h @ t[p + "k"].T).view(T, H, D)
    v = silu(h @ t[p + "v"].T).view(T, H, Dv)
    o = decayed_outer_products(q, k, v, torch.tensor(m["decay"], dtype=F64)).reshape(T, H * Dv)
    return (over_rms(o, eps) * t[p + "norm"] * torch.sigmoid(h @ t[p + "g"].T)) @ t[p + "o"].T


def positive_part(u: torch.Tensor) -> torch.Tensor:
    """A candidate that is positive and continuous: u + 1/2 from zero on, sigmoid(u) below."""
    return torch.where(u >= 0, u + 0.5, torch.sigmoid(u))


def gated_average(z: torch.Tensor, c: torch.Tensor) -> torch.Tensor:
    """S <- (1 - z) S + z c over the rows, from zeros."""
    S, out = torch.zeros_like(c[0]), torch.zeros_like(c)
    for i in range(c.shape[0]):
        S = (1.0 - z[i]) * S + z[i] * c[i]
        out[i] = S
    return out


def mingru_mixer(h: torch.Tensor, t: Dict[str, torch.Tensor], p: str) -> torch.Tensor:
    z = torch.sigmoid(h @ t[p + "z"].T + t[p + "z.b"])
    c = positive_part(h @ t[p + "x"].T + t[p + "x.b"])
    return (gated_average(z, c) * silu(h @ t[p + "g"].T)) @ t[p + "o"].T


# -- feed-forward and output -----------------------------------------------------------------------------
def poly_norm(z: torch.Tensor, coef: torch.Tensor, eps: float) -> torch.Tensor:
    a, b, c, e = (coef[i] for i in range(4))
    return a * over_rms(z, eps) + b * over_rms(z ** 2, eps) + c * over_rms(z ** 3, eps) + e


def dense_ff(h: torch.Tensor, t: Dict[str, torch.Tensor], p: str, eps: float) -> torch.Tensor:
    return poly_norm(h @ t[p + "up"].T, t[p + "act"], eps) @ t[p + "down"].T


def soft_cap(y: torch.Tensor, cap: float) -> torch.Tensor:
    return cap * torch.tanh(y / cap)


def forward(model: dict, tokens: List[int], streams: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab] of a whole sequence; `streams` collects the residual stream after every layer."""
    cfg, t = model["config"], model["tensors"]
    eps = cfg["norm"]["eps"]
    x = embedding(tokens, t["embed"], cfg["embedding"]["scale"])
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.mix.", layer["mixer"]
        h = stream_norm(x, t[f"l{i}.norm1"], eps)
        if layer["type"] == "attention":
            x = x + attention_mixer(h, t, p, m, eps)
        elif layer["type"] == "lightning":
            x = x + lightning_mixer(h, t, p, m, eps)
        elif layer["type"] == "mingru":
            x = x + mingru_mixer(h, t, p)
        else:
            raise ValueError(layer["type"])
        if layer.get("mlp") is not None:
            x = x + dense_ff(stream_norm(x, t[f"l{i}.norm2"], eps), t, f"l{i}.mlp.", eps)
        if streams is not None:
            streams.append(x.clone())
    y = stream_norm(x, t["final.norm"], eps) @ t["embed"].T * cfg["logit_scale"]
    return soft_cap(y, cfg["logit_softcap"])
