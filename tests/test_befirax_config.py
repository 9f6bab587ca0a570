"""Befirax without a GPU: the configuration's round trip and errors, tensor names and shapes, cache and state requests,
entries of the run order that read another layer's pages, the plain implementation against closed forms; and that each
mechanism, left out or moved by one, shifts the plain model's logits by far more than the tests' tolerance."""
from __future__ import annotations

import copy
import dataclasses
import math

import pytest
import torch

from serve_amd import ops
from serve_amd.cache.storage import group_windows
from serve_amd.config.befirax import BefiraxConfig
from serve_amd.config.llama import ConfigError
from serve_amd.models.befirax import build_befirax_spec
from serve_amd.models.model import Model
from serve_amd.parts.base import LayerCache
from serve_amd.parts.standard import rope_inverse_frequencies
from serve_amd.registry import get_part, load_config
from serve_amd.weights.loader import check_against
from serve_amd.weights.safetensors_io import CheckpointReader
from tests import befirax_models as bm
from tests.plain import befirax_plain as bp

F64 = torch.float64


@pytest.mark.parametrize("name", list(bm.MODELS))
def test_config_round_trip(name):
    cfg = bm.MODELS[name][0]
    d = cfg.to_hf_dict()
    assert d["architecture"] == "Befirax"
    again = BefiraxConfig.from_hf_dict(d)
    assert again == cfg and again.to_hf_dict() == d


def test_optional_keys_may_be_absent():
    d = bm.BA.to_hf_dict()
    del d["layers"][0]["mixer"]["rot"], d["layers"][0]["mixer"]["conv"], d["layers"][2]["mixer"]["rot"], d["layers"][2]["mlp"]
    del d["layers"][1]["mixer"]["mask"], d["layers"][0]["mlp"]["router"]["identity"]
    cfg = BefiraxConfig.from_hf_dict(d)
    assert cfg.layers[0].mixer.rot is None and cfg.layers[0].mixer.conv == 0 and cfg.layers[1].mixer.window is None
    assert cfg.layers[0].mlp.identity == 0 and cfg.layers[2].mlp is None
    model = Model(build_befirax_spec(cfg))
    names = {r.checkpoint_name: r.shape for r in model.weight_requests()}
    assert "l0.mix.q.conv" not in names and names["l0.mlp.router"] == (5, 64) and "l2.norm2" not in names
    assert model.state_requests()[0] is None and model.cache_requests()[1].retention is None


@pytest.mark.parametrize("change,message", [
    (lambda d: d["layers"][0].__setitem__("type", "other"), "not supported"),
    (lambda d: d["layers"][0]["mixer"].__setitem__("kv_heads", 3), "multiple"),
    (lambda d: d["layers"][0]["mixer"]["rot"].__setitem__("dims", 26), "fit"),
    (lambda d: d["layers"][0]["mixer"]["rot"].__setitem__("dims", 7), "even"),
    (lambda d: d["layers"][0]["mixer"].pop("diff"), "lacks"),
    (lambda d: d["layers"][0]["mixer"].__setitem__("conv", -1), "positive"),
    (lambda d: d["layers"][1]["mixer"]["mask"].__setitem__("size", 0), "positive"),
    (lambda d: d["layers"][1]["mixer"].__setitem__("rot_dim", 16), "whole rotated part"),
    (lambda d: d["layers"][2]["mixer"].__setitem__("kv_from", 2), "earlier"),
    (lambda d: d["layers"][2]["mixer"].__setitem__("kv_from", 1), "earlier"),
    (lambda d: d["layers"][2]["mixer"].__setitem__("heads", 2), "that layer's"),
    (lambda d: d["layers"][2]["mixer"]["rot"].__setitem__("base", 7.0), "that layer's"),
    (lambda d: d["layers"][3]["mixer"].__setitem__("groups", 3), "multiple"),
    (lambda d: d["layers"][0]["mlp"].__setitem__("kind", "other"), "not supported"),
    (lambda d: d["layers"][0]["mlp"]["router"].__setitem__("top", 8), "top"),
    (lambda d: d["layers"][0]["mlp"]["router"].__setitem__("identity", -1), "top"),
    (lambda d: d["layers"][0]["mlp"].pop("expert"), "lacks"),
    (lambda d: d.__setitem__("streams", 0), "positive"),
    (lambda d: d.pop("streams"), "lacks"),
])
def test_config_errors(change, message):
    d = copy.deepcopy(bm.BA.to_hf_dict())
    change(d)
    with pytest.raises(ConfigError, match=message):
        BefiraxConfig.from_hf_dict(d)


def test_tensor_names_cache_and_state():
    spec = build_befirax_spec(bm.BA)
    model = Model(spec)
    names = {r.checkpoint_name: r.shape for r in model.weight_requests() if not r.alias_only}
    assert names["embed"] == (150, 64) and names["final.norm"] == (64,) and "head" not in names
    assert names["l0.mix.q"] == (192, 64) and names["l0.mix.k"] == (96, 64) and names["l0.mix.v"] == (80, 64)
    assert names["l0.mix.q.b"] == (192,) and names["l0.mix.v.conv"] == (80, 3) and names["l0.mix.lq2"] == (24,)
    assert names["l0.mix.g"] == (160, 64) and names["l0.mix.o"] == (64, 160) and names["l0.mix.o.b"] == (64,)
    assert names["l0.mlp.router"] == (7, 64) and names["l0.mlp.correction"] == (7,) and names["l0.mlp.e4.down"] == (64, 32)
    assert "l0.mlp.e5.gate" not in names
    assert names["l0.hc1.in"] == (4,) and names["l0.hc2.mix"] == (4, 4) and "l2.hc2.mix" not in names
    assert names["l1.mix.q"] == (72, 64) and names["l1.mix.dkv"] == (48, 64) and names["l1.mix.g"] == (3, 64)
    assert names["l2.mix.q.conv"] == (192, 2) and "l2.mix.k" not in names and "l2.mix.v.conv" not in names
    assert names["l3.mix.in"] == (2 * 64 + 2 * 2 * 24 + 4, 64) and names["l3.mix.norm"] == (64,)
    creq, sreq = model.cache_requests(), model.state_requests()
    assert [None if c is None else c.retention for c in creq] == [None, 10, None, None, 5]
    # one key/value head a group: the two maps' keys side by side, the values once
    assert [t.shape for t in creq[0].tensors] == [(2, 48), (2, 48)] and creq[2] is None
    assert sreq[0].shape == (2 * (192 + 96 + 80),) and sreq[2].shape == (192,) and sreq[1] is None and sreq[4] is None
    assert group_windows(creq) == [None, 5, 10]
    # a step that reads layer 0's pages twice counts them twice
    assert sum(n for n, w in model.cache_elements_per_token() if w is None) == 2 * 2 * 96
    assert model.graph_safe()


def test_run_order_reads_another_layers_pages():
    spec = build_befirax_spec(bm.BA)
    order = spec.run_order
    assert [(e.cache, e.writes_cache, e.reads_pages_of) for e in order] == [(0, True, None), (1, True, None), (2, False, 0),
                                                                         (3, True, None), (4, True, None)]
    bad = dataclasses.replace(spec, run_order=[dataclasses.replace(order[2], reads_pages_of=1)] + order[:2] + order[3:])
    with pytest.raises(ValueError, match="before anything has written"):
        Model(bad)
    bad = dataclasses.replace(spec, run_order=order[:2] + [dataclasses.replace(order[2], writes_cache=True)] + order[3:])
    with pytest.raises(ValueError, match="does not write"):
        Model(bad)
    bad = dataclasses.replace(spec, run_order=order[:1] + [dataclasses.replace(order[1], writes_cache=False, reads_pages_of=0)] + order[2:])
    with pytest.raises(ValueError, match="keeps keys of its own"):
        Model(bad)
    a = LayerCache(group=1, pages={"k": torch.zeros(1)}, page_size=4, state=torch.zeros(2))
    b = LayerCache(state=torch.ones(3))
    c = a.with_state_of(b)
    assert c.group == 1 and c.pages is a.pages and c.page_size == 4 and c.state is b.state


def test_a_folder_loads_by_name_and_reports_what_does_not_fit(tmp_path):
    folder = bm.make_folder(tmp_path, "BC")
    arch, cfg = load_config(folder)
    assert arch.name == "Befirax" and cfg == bm.BC
    model = Model(arch.build_spec(cfg))
    assert len(check_against(model, CheckpointReader(folder))) == len(model.weight_requests())


def test_parts_refuse_what_they_do_not_compute():
    base = dict(hidden_size=32, num_heads=2, num_kv_heads=1, dim=16, vdim=16, scale=0.2, eps=1e-5, diff=0.3)
    att = get_part("mixer", "differential_attention")
    with pytest.raises(ValueError, match="taps"):
        att(**base, conv=ops.CONV_ATTENTION_MAX_TAPS + 1)
    with pytest.raises(ValueError, match="multiple"):
        att(**dict(base, num_kv_heads=3))
    with pytest.raises(ValueError, match="up to"):
        att(**dict(base, dim=400))
    with pytest.raises(ValueError, match="streams"):
        get_part("stream_weights", "hyper_connection")(ops.STREAM_MIX_MAX_STREAMS + 1)
    moe = get_part("feed_forward", "routed_experts")
    with pytest.raises(ValueError, match="top"):
        moe(32, 4, 7, 8, identity=2)
    with pytest.raises(ValueError, match="correction"):
        moe(32, 4, 2, 8, correction=True)
    with pytest.raises(ValueError, match="output"):
        moe(32, 4, 2, 8, identity=1, weight_inputs=True)
    assert moe(32, 4, 2, 8).leaves_rows and not moe(32, 4, 2, 8, shared_size=16).leaves_rows
    assert not moe(32, 12, 9, 8).leaves_rows
    with pytest.raises(ValueError, match="out_gate"):
        get_part("mixer", "latent_attention")(32, 2, 8, 4, 8, 16, 0.2, 1e-5, {"kind": "rope", "params": {}}, out_gate="row")


# ---------------------------------------------------------------------------------------------
# the plain implementation against closed forms
# ---------------------------------------------------------------------------------------------
def test_plain_streams():
    X = torch.tensor([[[1.0, 2.0]], [[10.0, 20.0]]], dtype=F64)              # two copies of one token of width 2
    assert bp.streams_in(X, torch.tensor([2.0, 0.5], dtype=F64)).tolist() == [[7.0, 14.0]]
    M = torch.tensor([[1.0, 3.0], [0.0, 2.0]], dtype=F64)                    # [from, to]
    y = torch.tensor([[100.0, -100.0]], dtype=F64)
    out = bp.streams_out(X, y, M, torch.tensor([1.0, 0.1], dtype=F64))
    assert out[0].tolist() == [[101.0, -98.0]]                               # 1 X_1 + 0 X_2 + y
    assert out[1].tolist() == [[33.0, 36.0]]                                 # 3 X_1 + 2 X_2 + 0.1 y, both from the old copies


def test_plain_convolution_and_rotation():
    u = torch.tensor([[1.0], [2.0], [3.0], [4.0]], dtype=F64)
    w = torch.tensor([[100.0, 10.0, 1.0]], dtype=F64)
    assert bp.causal_conv(u, w)[:, 0].tolist() == [1.0, 12.0, 123.0, 234.0]
    x = torch.arange(1.0, 6.0, dtype=F64).expand(4, 5)
    f1 = 10.0 ** (-2 / 4)
    c0, s0, c1, s1 = math.cos(3.0), math.sin(3.0), math.cos(3 * f1), math.sin(3 * f1)
    a, b = bp.rotate(x, 4, 10.0, "interleaved")[3], bp.rotate(x, 4, 10.0, "half")[3]
    assert torch.allclose(a, torch.tensor([1 * c0 - 2 * s0, 2 * c0 + 1 * s0, 3 * c1 - 4 * s1, 4 * c1 + 3 * s1, 5.0], dtype=F64))
    assert torch.allclose(b, torch.tensor([1 * c0 - 3 * s0, 2 * c1 - 4 * s1, 3 * c0 + 1 * s0, 4 * c1 + 2 * s1, 5.0], dtype=F64))
    f = rope_inverse_frequencies(4, 10.0, {"rope_type": "linear", "factor": 1.0})
    assert torch.allclose(f.double(), torch.tensor([1.0, f1], dtype=F64), rtol=1e-7)


def test_plain_softmax_and_window():
    v = torch.arange(1.0, 5.0, dtype=F64)
    s = torch.zeros(4, 4, dtype=F64)
    assert (bp.softmax_weights(s, None) @ v).tolist() == [1.0, 1.5, 2.0, 2.5]
    assert (bp.softmax_weights(s, 2) @ v).tolist() == [1.0, 1.5, 2.5, 3.5]
    assert (bp.softmax_weights(s, 1) @ v).tolist() == [1.0, 2.0, 3.0, 4.0]
    s[3, 1] = math.log(7.0)
    assert bp.softmax_weights(s, None)[3, 1].item() == pytest.approx(0.7)


def test_plain_differential_heads():
    """One token: both maps give v, so the head is (1 - lambda) v over its root mean square, times 1 - diff and the gate."""
    t = {"q": torch.ones(4, 2), "q.b": torch.zeros(4), "q.conv": torch.ones(4, 1), "k": torch.ones(4, 2), "k.b": torch.zeros(4),
         "k.conv": torch.ones(4, 1), "v": torch.tensor([[1.0, 0.0], [0.0, 1.0]]), "v.b": torch.tensor([1.0, 0.0]),
         "v.conv": 2.0 * torch.ones(2, 1), "lq1": torch.tensor([1.0, 0.0]), "lk1": torch.tensor([0.5, 3.0]),
         "lq2": torch.tensor([0.0, 1.0]), "lk2": torch.tensor([3.0, -0.25]), "g": torch.zeros(2, 2), "o": torch.eye(2),
         "o.b": torch.tensor([0.0, 10.0])}
    t = {k: v.to(F64) for k, v in t.items()}
    lam = math.exp(0.5) - math.exp(-0.25) + 0.4
    assert bp.diff_lambda(t, "", 0.4) == pytest.approx(lam)
    m = {"heads": 1, "kv_heads": 1, "dim": 2, "vdim": 2, "scale": 0.3, "diff": 0.4, "rot": {"dims": 2, "base": 10.0}}
    h = torch.tensor([[2.0, 1.0]], dtype=F64)
    out = bp.attention_mixer(h, t, "", m, 0.0, bp.attention_kv(h, t, "", m))
    v = torch.tensor([6.0, 2.0], dtype=F64)                                  # (convolved with one tap of 2)
    sign = 1.0 if lam < 1 else -1.0
    want = sign * v / math.sqrt((36 + 4) / 2) * 0.6 * 0.5 + torch.tensor([0.0, 10.0], dtype=F64)
    assert torch.allclose(out[0], want)


def test_plain_router_and_identity_experts():
    z = torch.tensor([[2.0, 1.0, 0.0, -1.0]], dtype=F64)
    s = torch.softmax(z, -1)[0]
    t = {"router": torch.eye(4, dtype=F64), "correction": torch.tensor([0.0, -1.0, 0.0, 1.0], dtype=F64)}
    ids, w = bp.route(z, t, "", 2)
    assert ids.tolist() == [[3, 0]]                                          # chosen with the correction ...
    assert torch.allclose(w[0], torch.stack([s[3], s[0]]) / (s[3] + s[0]))   # ... weighted without it
    # outputs 2 and 3 are identity experts
    t.update({f"e{e}.{n}": torch.zeros(4, 4, dtype=F64) for e in (0, 1) for n in ("gate", "up", "down")})
    out = bp.experts_ff(z, t, "", {"router": {"experts": 2, "top": 2}})
    assert torch.allclose(out, z * (s[3] / (s[3] + s[0])))


def test_plain_state_space_of_one_head():
    """Constant inputs: the state is a geometric sum."""
    a_log, dtb = -0.3, 0.2
    t = {"in": torch.tensor([[1.0], [1.0], [1.0], [1.0], [0.0]]), "conv": torch.ones(3, 1), "conv.b": torch.zeros(3),
         "dt_bias": torch.tensor([dtb]), "A_log": torch.tensor([a_log]), "D": torch.tensor([0.5]), "norm": torch.ones(1),
         "o": torch.ones(1, 1)}
    t = {k: v.to(F64) for k, v in t.items()}
    m = {"heads": 1, "vdim": 1, "state": 1, "groups": 1, "norm_groups": 1}
    h = torch.full((3, 1), 2.0, dtype=F64)
    out = bp.state_space_mixer(h, t, "", m, 1.0)[:, 0]
    x = 2.0 / (1 + math.exp(-2.0))
    dt = math.log1p(math.exp(dtb))
    a = math.exp(-math.exp(a_log) * dt)
    for n in range(3):
        S = dt * x * x * sum(a ** k for k in range(n + 1))
        y = (S * x + 0.5 * x) * x
        assert out[n].item() == pytest.approx(y / math.sqrt(y * y + 1.0))


def test_every_mechanism_shows_in_the_plain_logits(tmp_path):
    """Leaving a mechanism out, or moving an edge by one, moves the plain model's logits by 150 times the float32
    tolerance and more: a fault of that kind in the engine cannot hide behind the tolerance."""
    folder = bm.make_folder(tmp_path, "BAsharp", config=bm.BA, seed=3, scales=bm.SHARP)
    cfg, weights = bm.plain_config(folder), bm.plain_weights(folder)
    tokens = [(7 * i * i + 3 * i + 1) % 150 for i in range(40)]
    want = bm.plain_logits(folder, tokens)

    def moved(config=None, tensors=None, fn=None):
        saved = {n: getattr(bp, n) for n in (fn or {})}
        for n, f in (fn or {}).items():
            setattr(bp, n, f)
        try:
            got = bm.plain_logits(folder, tokens, config, tensors)
        finally:
            for n, f in saved.items():
                setattr(bp, n, f)
        return bm.row_distance(got, want)[-12:].max().item()

    def changed(path, value):
        c = copy.deepcopy(cfg)
        at = c
        for k in path[:-1]:
            at = at[k]
        at[path[-1]] = value
        return moved(c)

    bound = 150 * bm.TOLERANCE["float32"]
    for layer, size in ((1, 9), (1, 11), (4, 4), (4, 6)):
        assert changed(("layers", layer, "mixer", "mask", "size"), size) > bound, f"window of layer {layer} at {size}"
    for layer in (0, 2):
        assert changed(("layers", layer, "mixer", "diff"), 0.5) > bound
        assert changed(("layers", layer, "mixer", "scale"), 0.6) > bound
    assert changed(("layers", 0, "mixer", "rot", "dims"), 10) > bound
    assert changed(("layers", 1, "mixer", "rot", "base"), 500.0) > bound
    assert changed(("layers", 0, "mlp", "router", "top"), 3) > bound
    assert changed(("norm", "eps"), 1.0) > bound
    for name in ("l0.mix.q.b", "l0.mix.k.b", "l0.mix.v.b", "l0.mix.o.b", "l2.mix.q.b", "l0.mix.lq1", "l2.mix.lk2", "l0.mix.g",
                 "l1.mix.g", "l0.mlp.correction", "l3.mix.conv.b", "l3.mix.D", "l3.mix.dt_bias"):
        w = dict(weights)
        w[name] = torch.zeros_like(w[name])
        assert moved(tensors=w) > bound, name
    for name, col in (("l0.mix.q.conv", 0), ("l0.mix.k.conv", 1), ("l0.mix.v.conv", 0), ("l2.mix.q.conv", 0), ("l3.mix.conv", 0)):
        w = dict(weights)
        w[name] = w[name].clone()
        w[name][:, col] = 0
        assert moved(tensors=w) > bound, f"tap {col} of {name}"
    for name in ("l0.norm1", "l0.norm2", "l1.mix.dkv.norm", "final.norm", "l3.mix.norm"):
        w = dict(weights)
        w[name] = torch.ones_like(w[name])
        assert moved(tensors=w) > bound, name
    w = dict(weights)                                                         # the matrix read as [to, from]
    w["l1.hc1.mix"] = w["l1.hc1.mix"].T.contiguous()
    assert moved(tensors=w) > bound
    out = bp.streams_out

    def one_after_another(X, y, M, b):
        X = X.clone()
        for t in range(X.shape[0]):
            X[t] = sum(M[s, t] * X[s] for s in range(X.shape[0])) + b[t] * y
        return X
    assert moved(fn={"streams_out": one_after_another}) > bound
    assert moved(fn={"streams_out": lambda X, y, M, b: out(X, y, M, torch.ones_like(b))}) > bound
    conv, rot = bp.causal_conv, bp.rotate
    assert moved(fn={"causal_conv": lambda u, w: conv(torch.cat([torch.zeros_like(u[:20]), u[20:]]), w)}) > bound     # a lost state
    assert moved(fn={"rotate": lambda x, d, b, l: rot(x, d, b, "half")}) > bound
    assert moved(fn={"diff_lambda": lambda t, p, d: 0.0}) > bound                                                     # one map alone

    def rotated_first(h, t, p, m):                       # (the convolution behind the rotation instead of before it)
        T, G = h.shape[0], m["kv_heads"]
        k = rot((h @ t[p + "k"].T + t[p + "k.b"]).view(T, G, 2, m["dim"]), m["rot"]["dims"], m["rot"]["base"], "interleaved")
        return conv(k.reshape(T, -1), t[p + "k.conv"]).view(T, G, 2, m["dim"]), bp.projected(h, t, p + "v").view(T, G, m["vdim"])
    assert moved(fn={"attention_kv": rotated_first}) > bound

    def no_identity(h, t, p, c):
        ids, w = bp.route(h, t, p, c["router"]["top"])
        E = c["router"]["experts"]
        y = torch.zeros_like(h)
        for n in range(h.shape[0]):
            for k in range(ids.shape[1]):
                e = int(ids[n, k])
                if e < E:
                    q = f"{p}e{e}."
                    y[n] += w[n, k] * (t[q + "down"] @ (bp.silu(t[q + "gate"] @ h[n]) * (t[q + "up"] @ h[n])))
        return y
    assert moved(fn={"experts_ff": no_identity}) > bound
