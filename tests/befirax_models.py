"""Small Befirax models for the tests, their folders with random weights, and comparisons of the engine's logits with
the plain implementation's (tests/plain/befirax_plain.py).

The models differ in every size and option:
  BA  width 64, 4 streams; attention 4 heads on 2, maps of 24 with 8 rotated dims, values 40 (a cache head of 48), 3 taps,
      experts top 2 of 5 + 2 identity; latent attention 3 heads of 16 + 8, values 24, latent 40, a window of 10, top 3 of
      4 + 1; attention that reads layer 0's keys and values (2 taps, other constants), no feed-forward; a state-space layer of
      4 heads 24 x 16 in 2 groups, 4 taps, no feed-forward; latent attention 2 heads, a window of 5 (pages hold 8)
  BB  width 96, 2 streams; a state-space layer first; attention 6 heads on 3, maps of 16 rotated whole, values 32 (twice the
      map: no padding), 4 taps; two layers that read it, one behind the other; latent attention with a window of 33; top 4
      of 6 without identity experts and top 4 of 3 + 3
  BC  width 50 (no multiple of 8), 3 streams, vocabulary 101; attention 3 heads on 3, maps of 6, values 7, one tap; 2 heads
      of 6 + 4, values 5, latent 9, a window of 4; a state-space layer of 3 heads 6 x 5 in 3 groups and 3 norm groups, 2 taps
  BD  sizes above what the fast kernels take: maps of 72 (a cache head of 144), 5 taps, 5 streams, a latent row of 200 + 16,
      states of 136, top 9 of 10 + 2
  BE  values that are 1: one stream, one head, one tap, a window of one, one expert and one identity expert, one group
  BF  maps of 32, values 64, 2 taps, 8 heads on 1; no layer but attention, the last two read the first
"""
from __future__ import annotations

import json
import os
from typing import Dict, List, Optional

import torch

from serve_amd.config.befirax import (BefiraxConfig, BefiraxLayerConfig, DifferentialAttentionConfig, IdentityMoeConfig,
                                      PlainRotConfig, WindowedLatentConfig)
from serve_amd.config.kotipel import StateSpaceMixerConfig
from serve_amd.weights.loader import write_random_model
from tests.plain import befirax_plain

L = BefiraxLayerConfig
ATT, LAT, SSM, MOE, ROT = (DifferentialAttentionConfig, WindowedLatentConfig, StateSpaceMixerConfig, IdentityMoeConfig,
                           PlainRotConfig)

BA = BefiraxConfig(vocab=150, width=64, eps=1e-5, streams=4, layers=(
    L(ATT(4, 2, 24, 40, 0.25, 0.4, 3, ROT(100.0, 8)), MOE(5, 2, 2, 32)),
    L(LAT(3, 16, 8, 24, 40, 0.2, ROT(50.0, 8), 10), MOE(4, 1, 3, 40)),
    L(ATT(4, 2, 24, 40, 0.18, 0.6, 2, ROT(100.0, 8), 0), None),
    L(SSM(4, 16, 24, 2, 4, 1), None),
    L(LAT(2, 8, 16, 16, 24, 0.3, ROT(300.0, 16), 5), MOE(3, 1, 1, 24)),
))

BB = BefiraxConfig(vocab=211, width=96, eps=1e-6, streams=2, layers=(
    L(SSM(6, 32, 16, 3, 3, 2), MOE(6, 0, 4, 40)),
    L(ATT(6, 3, 16, 32, 0.3, 0.2, 4, ROT(1000.0, 16)), None),
    L(ATT(6, 3, 16, 32, 0.35, 0.5, 4, ROT(1000.0, 16), 1), MOE(3, 3, 4, 24)),
    L(LAT(4, 16, 16, 8, 48, 0.25, ROT(10000.0, 16), 33), None),
    L(ATT(6, 3, 16, 32, 0.25, 0.3, 2, ROT(1000.0, 16), 1), None),
))

BC = BefiraxConfig(vocab=101, width=50, eps=1e-4, streams=3, layers=(
    L(LAT(2, 6, 4, 5, 9, 0.4, ROT(20.0, 4), 4), MOE(5, 2, 3, 9)),
    L(ATT(3, 3, 6, 7, 0.5, 0.35, 1, ROT(50.0, 4)), MOE(2, 1, 2, 11)),
    L(SSM(3, 5, 6, 3, 2, 3), MOE(4, 4, 4, 13)),
    L(ATT(3, 3, 6, 7, 0.4, 0.1, 3, ROT(50.0, 4), 1), None),
))

BD = BefiraxConfig(vocab=120, width=64, eps=1e-5, streams=5, layers=(
    L(ATT(2, 1, 72, 24, 0.12, 0.45, 5, ROT(5000.0, 36)), MOE(10, 2, 9, 16)),
    L(LAT(2, 24, 16, 16, 200, 0.12, ROT(200.0, 16), 40), MOE(4, 1, 2, 20)),
    L(SSM(2, 24, 136, 1, 4, 2), None),
    L(ATT(2, 1, 72, 24, 0.1, 0.3, 3, ROT(5000.0, 36), 0), None),
))

BE = BefiraxConfig(vocab=77, width=32, eps=1e-5, streams=1, layers=(
    L(ATT(1, 1, 16, 16, 0.4, 0.5, 1, ROT(10.0, 2)), MOE(1, 1, 1, 8)),
    L(LAT(1, 8, 2, 8, 16, 0.4, ROT(10.0, 2), 1), MOE(1, 0, 1, 8)),
    L(SSM(1, 16, 8, 1, 1, 1), None),
    L(ATT(1, 1, 16, 16, 0.4, 0.0, 1, ROT(10.0, 2), 0), MOE(1, 1, 2, 8)),
))

BF = BefiraxConfig(vocab=130, width=64, eps=1e-5, streams=3, layers=(
    L(ATT(8, 1, 32, 64, 0.2, 0.25, 2, ROT(500.0, 24)), None),
    L(ATT(8, 1, 32, 64, 0.25, 0.55, 4, ROT(500.0, 24), 0), MOE(4, 2, 2, 24)),
    L(ATT(8, 1, 32, 64, 0.15, 0.7, 1, ROT(500.0, 24), 0), None),
))

MODELS = {"BA": (BA, 3), "BB": (BB, 11), "BC": (BC, 5), "BD": (BD, 6), "BE": (BE, 7), "BF": (BF, 8)}

# the table at a scale at which the stream and the logits are of order one; corrections that change many choices
BASE = {r"^embed$": 14.0, r"mlp\.correction$": 6.0, r"mix\.o$": 2.0, r"mlp\.e\d+\.down$": 2.0}

# queries and keys drawn wider: scores of order one and more, so that the softmax picks keys instead of averaging them
# and a key lost or let in at a window's edge moves the logits by far more than the bfloat16 tolerance
SHARP = {r"mix\.(q|k|uk)$": 4.0, r"^l1\.mix\.o$": 3.0, r"^l4\.mix\.o$": 8.0, r"mix\.l[qk][12]$": 2.5}

# the latent layers' scores wider and their outputs stronger: enough for a window's edge to show, without turning the
# softmax into a choice that bfloat16 may make otherwise
EDGES = {r"^l[14]\.mix\.q$": 2.0, r"^l4\.mix\.o$": 4.0, r"^l1\.mix\.o$": 2.0}

# per row of logits: root mean square of the difference over that of the row.  float32: a few ulp of the largest
# intermediate; bfloat16: 8 bits of mantissa at every product's input
TOLERANCE = {"float32": 2e-4, "bfloat16": 0.08}


def make_folder(tmp_path, name: str, config: Optional[BefiraxConfig] = None, seed=None, scales=None) -> str:
    cfg, s = MODELS.get(name, (config, seed))
    folder = os.path.join(str(tmp_path), f"befirax_{name}")
    if not os.path.isdir(folder):
        write_random_model(folder, cfg if config is None else config, s if seed is None else seed,
                           scales=dict(BASE, **(scales or {})))
    return folder


def plain_weights(folder: str) -> Dict[str, torch.Tensor]:
    from safetensors.torch import load_file
    return load_file(os.path.join(folder, "model.safetensors"))


def plain_config(folder: str) -> dict:
    with open(os.path.join(folder, "config.json")) as f:
        return json.load(f)


def plain_logits(folder: str, tokens: List[int], config: Optional[dict] = None,
                 weights: Optional[Dict[str, torch.Tensor]] = None) -> torch.Tensor:
    w = weights or plain_weights(folder)
    model = {"config": config or plain_config(folder), "tensors": {k: v.double() for k, v in w.items()}}
    return befirax_plain.forward(model, tokens)


def row_distance(got: torch.Tensor, want: torch.Tensor) -> torch.Tensor:
    """Per row: the root mean square of the difference (its mean taken off) over that of the wanted row."""
    got, want = got.detach().double().cpu(), want.detach().double().cpu()
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    w = want - want.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / w.pow(2).mean(-1).sqrt().clamp_min(1e-12)


def assert_rows_close(got: torch.Tensor, want: torch.Tensor, dtype: str, what: str = "") -> None:
    assert got.shape == want.shape, f"{what}: shape {tuple(got.shape)} vs {tuple(want.shape)}"
    dist = row_distance(got, want)
    bad = (dist > TOLERANCE[dtype]) | ~torch.isfinite(dist)
    if bad.any():
        i = int(bad.nonzero()[0])
        raise AssertionError(f"{what}: {int(bad.sum())} of {bad.numel()} rows differ; first row {i}: distance "
                             f"{dist[i].item():.3g}, allowed {TOLERANCE[dtype]:.3g}; worst {dist.max().item():.3g}")


SHAKE_RUNS, SHAKE = 6, 2.0 ** -8
CLOSE_CALL = 0.005         # shares plus correction of the last chosen and the first not chosen, apart


def shaky_rows(folder: str, tokens: List[int], want: torch.Tensor) -> torch.Tensor:
    """Rows of the plain model's logits that rest on a close call (a router's choice between two experts whose scores
    nearly tie moves the token's own row and, through keys, values and states, rows behind it).  Found by running the
    plain model several times more with every tensor disturbed by a relative 2^-8 (what rounding its products' operands
    to bfloat16 adds up to): rows that move by a quarter of the tolerance; and tokens whose own choice is closer than CLOSE_CALL."""
    out = torch.zeros(len(tokens), dtype=torch.bool)
    route = befirax_plain.route

    def watched(h, t, p, top):
        s = torch.sort(torch.softmax(h @ t[p + "router"].T, dim=-1) + t[p + "correction"], dim=-1, descending=True).values
        if top < s.shape[1]:
            out.logical_or_(s[:, top - 1] - s[:, top] < CLOSE_CALL)
        return route(h, t, p, top)
    try:
        befirax_plain.route = watched
        befirax_plain.forward({"config": plain_config(folder), "tensors": {k: v.double() for k, v in plain_weights(folder).items()}},
                              tokens)
    finally:
        befirax_plain.route = route
    for k in range(SHAKE_RUNS):
        g = torch.Generator().manual_seed(7 + 1000 * k)
        W = {n: v.double() * (1 + SHAKE * (2 * torch.rand(v.shape, generator=g, dtype=torch.float64) - 1))
             for n, v in plain_weights(folder).items()}
        moved = row_distance(befirax_plain.forward({"config": plain_config(folder), "tensors": W}, tokens), want)
        out |= moved > 0.25 * TOLERANCE["bfloat16"]
    return out


def assert_matches_plain(got: torch.Tensor, folder: str, tokens: List[int], dtype: str, what: str = "", rows=None) -> None:
    """`got`: the engine's logits for all of `tokens`, or for the places `rows` among them.  float32: every row.
    bfloat16: the rows that are well conditioned in the plain model (`shaky_rows`; in all but the shortest sequences there must be plenty of them)."""
    want = plain_logits(folder, tokens)
    keep = None
    if dtype == "bfloat16":
        keep = ~shaky_rows(folder, tokens, want)
    if rows is not None:
        want = want[rows]
        keep = None if keep is None else keep[rows]
    assert got.shape == want.shape, f"{what}: shape {tuple(got.shape)} vs {tuple(want.shape)}"
    got = got.detach().cpu()
    if keep is not None:
        assert len(keep) < 20 or keep.float().mean().item() >= 0.4, f"{what}: too many rows rest on close calls"
        assert torch.isfinite(got).all()
        got, want = got[keep], want[keep]
    assert_rows_close(got, want, dtype, what)


def engine_for(folder: str, dtype: str, num_pages=64, page_size=8, max_requests=4, **kw):
    from serve_amd.config.engine import EngineConfig
    from serve_amd.engine.engine import Engine
    cfg = EngineConfig(dtype=dtype, page_size=page_size, num_pages=num_pages, max_context=num_pages * page_size,
                       max_requests=max_requests, max_tokens_per_step=4096, prefill_chunk=4096, **kw)
    return Engine.from_folder(folder, cfg)


def run_portions(engine, rid, tokens, portions):
    """Feed `tokens` in the given portion sizes, wanting every position; returns [len, V]."""
    from serve_amd.engine.batch import Segment
    assert sum(portions) == len(tokens)
    assert engine.runner.admit(rid)
    rows, at = [], 0
    for n in portions:
        rows.append(engine.step([Segment(rid, tokens[at: at + n], list(range(n)))]))
        at += n
    engine.runner.release(rid)
    return torch.cat(rows, dim=0)
