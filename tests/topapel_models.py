"""Small Topapel models for the tests, their folders with random weights, and comparisons of the engine's logits with
the plain implementation's (tests/plain/topapel_plain.py).

The models differ in every size and option:
  TA  width 64; attention 4 heads on 2 of 32, half of the dims rotated with a third of the frequency, chunks of 10, with a
      feed-forward; a gated average of 80 channels with a feed-forward; a linear attention of 3 heads 24 x 40, one of which
      never decays, without; attention 2 heads on 1 of 24 (a cache head of 32), all dims rotated, chunks of 5 (pages hold 8)
  TB  width 96; a linear attention first, 2 heads 16 x 72; attention 6 on 3 of 16 that sees everything, without rotation;
      a gated average of 300 channels; attention 5 on 5 of 16 in chunks of 16; no two layers alike in having a feed-forward
  TC  width 50 (no multiple of 8), vocabulary 101; attention 3 on 3 of 10, 4 rotated dims, chunks of 33; 2 heads 6 x 5; a
      gated average of 37 channels; feed-forwards of 27, 11 and 9
  TD  sizes above what the matrix-core kernels take: attention heads of 136, linear-attention keys of 136, chunks of 40; a
      gated average of 1,100 channels; a feed-forward of 2,100
  TE  recurrent layers alone: nothing is kept per token
  TF  values that are 1: chunks of one position, one head, one channel, a decay of 1; and decays so fast that sixteen tokens
      leave the range of a float
"""
from __future__ import annotations

import json
import os
from typing import Dict, List, Optional

import torch

from serve_amd.config.topapel import (ChunkAttentionConfig, LightningConfig, LinearRotConfig, MinGruConfig, TopapelConfig,
                                      TopapelLayerConfig)
from serve_amd.weights.loader import write_random_model
from tests.plain import topapel_plain

L = TopapelLayerConfig
ATT, LIN, GRU, ROT = ChunkAttentionConfig, LightningConfig, MinGruConfig, LinearRotConfig

TA = TopapelConfig(vocab=150, width=64, eps=1e-5, embedding_scale=3.5, logit_scale=0.7, logit_softcap=6.0, layers=(
    L(ATT(4, 2, 32, 0.3, 10, ROT(100.0, 16, 3.0)), 96),
    L(GRU(80), 72),
    L(LIN(3, 24, 40, (0.5, 0.95, 1.0)), None),
    L(ATT(2, 1, 24, 0.35, 5, ROT(10000.0, 24, None)), None),
))

TB = TopapelConfig(vocab=211, width=96, eps=1e-6, embedding_scale=5.0, logit_scale=1.0, logit_softcap=7.0, layers=(
    L(LIN(2, 16, 72, (0.8, 0.999)), 120),
    L(ATT(6, 3, 16, 0.4, None, None), None),
    L(GRU(300), None),
    L(ATT(5, 5, 16, 0.5, 16, ROT(30.0, 16, 1.0)), 56),
))

TC = TopapelConfig(vocab=101, width=50, eps=1e-4, embedding_scale=2.5, logit_scale=1.3, logit_softcap=4.0, layers=(
    L(ATT(3, 3, 10, 0.6, 33, ROT(50.0, 4, 8.0)), 27),
    L(LIN(2, 6, 5, (0.9, 0.3)), 11),
    L(GRU(37), 9),
))

TD = TopapelConfig(vocab=120, width=64, eps=1e-5, embedding_scale=4.0, logit_scale=0.5, logit_softcap=10.0, layers=(
    L(ATT(2, 1, 136, 0.12, 40, ROT(5000.0, 64, 2.0)), None),
    L(LIN(2, 136, 24, (0.7, 0.97)), None),
    L(GRU(1100), 2100),
))

TE = TopapelConfig(vocab=90, width=48, eps=1e-5, embedding_scale=4.0, logit_scale=0.9, logit_softcap=8.0, layers=(
    L(GRU(64), 40),
    L(LIN(4, 8, 16, (0.6, 0.9, 0.99, 0.9999)), None),
))

TF = TopapelConfig(vocab=77, width=32, eps=1e-5, embedding_scale=3.0, logit_scale=1.0, logit_softcap=9.0, layers=(
    L(ATT(1, 1, 16, 0.4, 1, ROT(10.0, 2, 0.5)), None),
    L(LIN(1, 16, 16, (1.0,)), None),
    L(GRU(1), None),
    L(LIN(3, 16, 32, (1e-6, 1e-30, 0.004)), 20),
))

MODELS = {"TA": (TA, 3), "TB": (TB, 4), "TC": (TC, 5), "TD": (TD, 6), "TE": (TE, 7), "TF": (TF, 8)}

# the table at a scale at which the stream is of order one and the logits reach for the cap
BASE = {r"^embed$": 12.0}

# outputs drawn wider, so that what a single key or state adds shows in the logits
SHARP = {r"mix\.o$": 3.0, r"^l1\.mix\.o$": 4.0}

# per row of logits: root mean square of the difference over that of the row.  float32: a few ulp of the largest
# intermediate; bfloat16: 8 bits of mantissa at every product's input
TOLERANCE = {"float32": 2e-4, "bfloat16": 0.08}


def make_folder(tmp_path, name: str, config: Optional[TopapelConfig] = None, seed=None, scales=None) -> str:
    cfg, s = MODELS.get(name, (config, seed))
    folder = os.path.join(str(tmp_path), f"topapel_{name}")
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
    return topapel_plain.forward(model, tokens)


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
