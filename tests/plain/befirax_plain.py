"""A plain, slow implementation of the Befirax decoder in float64: one function per mechanism, whole sequences at a
time, no cache.  It shares no code with the package; the tests compare the engine with it.

    X_s = E[token]  for s = 1 .. streams                                     (X: streams x T x width)
    every sublayer f (a mixer, or a feed-forward) with its a [streams], M [streams, streams], b [streams]:
        u = sum_s a_s X_s;   y = f(N(u) w);   X_t <- sum_s M_st X_s + b_t y
    logits = E (N(sum_s X_s) w_final)

A model is a dict: {"config": the configuration as config.json holds it, "tensors": {name: float64 tensor}}.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch

F64 = torch.float64
Tensors = Dict[str, torch.Tensor]


def rms_norm(x: torch.Tensor, w: Optional[torch.Tensor], eps: float) -> torch.Tensor:
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if w is None else y * w


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def streams_in(X: torch.Tensor, a: torch.Tensor) -> torch.Tensor:
    """X [S, T, d] -> [T, d]"""
    out = torch.zeros_like(X[0])
    for s in range(X.shape[0]):
        out = out + a[s] * X[s]
    return out


def streams_out(X: torch.Tensor, y: torch.Tensor, M: torch.Tensor, b: torch.Tensor) -> torch.Tensor:
    """All streams at once from the old ones: M is indexed [from, to]."""
    S = X.shape[0]
    new = []
    for t in range(S):
        acc = b[t] * y
        for s in range(S):
            acc = acc + M[s, t] * X[s]
        new.append(acc)
    return torch.stack(new)


def causal_conv(u: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """u [T, C], w [C, taps] (its last column meets the current token); zeros before the first token."""
    T, taps = u.shape[0], w.shape[1]
    out = torch.zeros_like(u)
    for t in range(T):
        for j in range(taps):
            at = t - taps + 1 + j
            if at >= 0:
                out[t] += w[:, j] * u[at]
    return out


def rotate(x: torch.Tensor, dims: int, base: float, layout: str) -> torch.Tensor:
    """x [T, ..., D] at positions 0 .. T - 1: the first `dims` of D turned; `layout` 'interleaved' pairs (2i, 2i + 1),
    'half' pairs (i, i + dims / 2)."""
    n = dims // 2
    f = base ** (-2.0 * torch.arange(n, dtype=F64) / dims)
    a = torch.arange(x.shape[0], dtype=F64)[:, None] * f[None, :]
    a = a.view((x.shape[0],) + (1,) * (x.dim() - 2) + (n,))
    cos, sin = torch.cos(a), torch.sin(a)
    out = x.clone()
    first, second = (slice(0, dims, 2), slice(1, dims, 2)) if layout == "interleaved" else (slice(0, n), slice(n, dims))
    u, v = x[..., first], x[..., second]
    out[..., first] = u * cos - v * sin
    out[..., second] = v * cos + u * sin
    return out


def softmax_weights(s: torch.Tensor, window: Optional[int]) -> torch.Tensor:
    """s [T, T] scores of query i and key j -> weights over the keys 0 <= i - j (< window)."""
    i = torch.arange(s.shape[0])
    dist = i[:, None] - i[None, :]
    seen = dist >= 0
    if window is not None:
        seen &= dist < window
    s = s.masked_fill(~seen, -math.inf)
    e = torch.exp(s - s.max(-1, keepdim=True).values)
    return e / e.sum(-1, keepdim=True)


def diff_lambda(t: Tensors, p: str, diff: float) -> float:
    return float(torch.exp((t[p + "lq1"] * t[p + "lk1"]).sum()) - torch.exp((t[p + "lq2"] * t[p + "lk2"]).sum())) + diff


def projected(h: torch.Tensor, t: Tensors, name: str) -> torch.Tensor:
    """W h + b, then the convolution over time."""
    return causal_conv(h @ t[name].T + t[name + ".b"], t[name + ".conv"])


def attention_kv(h: torch.Tensor, t: Tensors, p: str, m: dict) -> Tuple[torch.Tensor, torch.Tensor]:
    """Keys [T, G, 2, dim] (convolved and rotated) and values [T, G, vdim] (convolved)."""
    T, G = h.shape[0], m["kv_heads"]
    k = projected(h, t, p + "k").view(T, G, 2, m["dim"])
    v = projected(h, t, p + "v").view(T, G, m["vdim"])
    return rotate(k, m["rot"]["dims"], m["rot"]["base"], "interleaved"), v


def attention_mixer(h: torch.Tensor, t: Tensors, p: str, m: dict, eps: float, kv) -> torch.Tensor:
    T, H, G, D, Dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    k, v = kv
    q = rotate(projected(h, t, p + "q").view(T, H, 2, D), m["rot"]["dims"], m["rot"]["base"], "interleaved")
    lam, diff = diff_lambda(t, p, m["diff"]), m["diff"]
    heads = []
    for i in range(H):
        g = i // (H // G)
        a = [softmax_weights((q[:, i, n] @ k[:, g, n].T) * m["scale"], None) @ v[:, g] for n in (0, 1)]
        heads.append(rms_norm(a[0] - lam * a[1], None, eps) * (1.0 - diff))
    o = torch.cat(heads, dim=-1) * torch.sigmoid(h @ t[p + "g"].T)
    return o @ t[p + "o"].T + t[p + "o.b"]


def latent_mixer(h: torch.Tensor, t: Tensors, p: str, m: dict, eps: float) -> torch.Tensor:
    T, H, D, R, Dv, rank = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (h @ t[p + "q"].T).view(T, H, D + R)
    z = h @ t[p + "dkv"].T
    c = rms_norm(z[:, :rank], t[p + "dkv.norm"], eps)
    kr = rotate(z[:, rank:], R, m["rot"]["base"], "half")
    qr = rotate(q[..., D:], R, m["rot"]["base"], "half")
    ku = (c @ t[p + "uk"].T).view(T, H, D)
    v = (c @ t[p + "uv"].T).view(T, H, Dv)
    gate = torch.sigmoid(h @ t[p + "g"].T)
    window = (m.get("mask") or {}).get("size")
    out = []
    for i in range(H):
        s = (q[:, i, :D] @ ku[:, i].T + qr[:, i] @ kr.T) * m["scale"]
        out.append(softmax_weights(s, window) @ v[:, i] * gate[:, i: i + 1])
    return torch.cat(out, dim=-1) @ t[p + "o"].T


def state_space_mixer(h: torch.Tensor, t: Tensors, p: str, m: dict, eps: float) -> torch.Tensor:
    T, H, P, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * P
    z, xbc, dt = (h @ t[p + "in"].T).split([inner, inner + 2 * G * N, H], dim=-1)
    xbc = silu(causal_conv(xbc, t[p + "conv"]) + t[p + "conv.b"])
    x = xbc[:, :inner].view(T, H, P)
    B = xbc[:, inner: inner + G * N].view(T, G, N)
    C = xbc[:, inner + G * N:].view(T, G, N)
    dt = torch.log1p(torch.exp(dt + t[p + "dt_bias"]))
    y = torch.zeros((T, H, P), dtype=F64)
    for i in range(H):
        g = i // (H // G)
        S = torch.zeros((N, P), dtype=F64)
        for n in range(T):
            S = torch.exp(-torch.exp(t[p + "A_log"][i]) * dt[n, i]) * S + dt[n, i] * torch.outer(B[n, g], x[n, i])
            y[n, i] = S.T @ C[n, g] + t[p + "D"][i] * x[n, i]
    y = y.view(T, inner) * silu(z)
    k = m["norm_groups"]
    y = rms_norm(y.view(T, k, inner // k), None, eps).reshape(T, inner) * t[p + "norm"]
    return y @ t[p + "o"].T


def route(h: torch.Tensor, t: Tensors, p: str, top: int) -> Tuple[torch.Tensor, torch.Tensor]:
    """(experts [T, top], weights [T, top]): chosen by the softmax's shares plus the correction, weighted by the shares."""
    s = torch.softmax(h @ t[p + "router"].T, dim=-1)
    ids = torch.topk(s + t[p + "correction"], top, dim=-1).indices
    w = torch.gather(s, 1, ids)
    return ids, w / (w.sum(-1, keepdim=True) + 1e-20)


def experts_ff(h: torch.Tensor, t: Tensors, p: str, c: dict) -> torch.Tensor:
    E, top = c["router"]["experts"], c["router"]["top"]
    ids, w = route(h, t, p, top)
    out = torch.zeros_like(h)
    for n in range(h.shape[0]):
        for k in range(top):
            e = int(ids[n, k])
            if e >= E:                                   # an identity expert
                y = h[n]
            else:
                q = f"{p}e{e}."
                y = t[q + "down"] @ (silu(t[q + "gate"] @ h[n]) * (t[q + "up"] @ h[n]))
            out[n] += w[n, k] * y
    return out


def forward(model: dict, tokens: List[int], stream_after: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab]; `stream_after` receives the sum of the streams after every layer."""
    cfg, t = model["config"], model["tensors"]
    eps = cfg["norm"]["eps"]
    x = t["embed"][torch.tensor(tokens)]
    X = torch.stack([x] * cfg["streams"])
    kept = {}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h = rms_norm(streams_in(X, t[p + "hc1.in"]), t[p + "norm1"], eps)
        if layer["type"] == "attention":
            j = m.get("kv_from")
            kept[i] = kept[j] if j is not None else attention_kv(h, t, p + "mix.", m)
            y = attention_mixer(h, t, p + "mix.", m, eps, kept[i])
        elif layer["type"] == "latent_attention":
            y = latent_mixer(h, t, p + "mix.", m, eps)
        else:
            y = state_space_mixer(h, t, p + "mix.", m, eps)
        X = streams_out(X, y, t[p + "hc1.mix"], t[p + "hc1.out"])
        if layer.get("mlp"):
            h = rms_norm(streams_in(X, t[p + "hc2.in"]), t[p + "norm2"], eps)
            X = streams_out(X, experts_ff(h, t, p + "mlp.", layer["mlp"]), t[p + "hc2.mix"], t[p + "hc2.out"])
        if stream_after is not None:
            stream_after.append(X.sum(0))
    return rms_norm(X.sum(0), t["final.norm"], eps) @ t["embed"].T
