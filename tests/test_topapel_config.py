"""Topapel without a GPU: the configuration's round trip and errors, tensor names and shapes, cache and state requests,
retention by chunks in the cache manager, and the plain implementation against closed forms; and that each mechanism,
left out or moved by one, shifts the plain model's logits by far more than the tests' tolerance."""
from __future__ import annotations

import copy
import math

import pytest
import torch

from serve_amd.cache.manager import FREED, CacheManager
from serve_amd.cache.retention import Chunks, first_seen, mean_seen, reach
from serve_amd.cache.storage import group_windows
from serve_amd.config.llama import ConfigError
from serve_amd.config.spec import PartSpec
from serve_amd.config.topapel import TopapelConfig
from serve_amd.models.model import Model
from serve_amd.models.topapel import build_topapel_spec
from serve_amd.parts.base import TokenCacheRequest, keys_seen
from serve_amd.parts.standard import rope_inverse_frequencies
from serve_amd.registry import get_part
from tests import topapel_models as tm
from tests.plain import topapel_plain as tp

F64 = torch.float64


@pytest.mark.parametrize("name", list(tm.MODELS))
def test_config_round_trip(name):
    cfg = tm.MODELS[name][0]
    d = cfg.to_hf_dict()
    assert d["architecture"] == "Topapel"
    again = TopapelConfig.from_hf_dict(d)
    assert again == cfg and again.to_hf_dict() == d


def test_optional_keys_may_be_absent():
    d = tm.TA.to_hf_dict()
    del d["layers"][0]["mixer"]["rot"]["scaling"], d["layers"][0]["mixer"]["mask"], d["layers"][3]["mixer"]["rot"]
    del d["layers"][3]["mixer"]["vdim"], d["layers"][2]["mlp"]
    d["layers"][1]["mlp"] = None
    cfg = TopapelConfig.from_hf_dict(d)
    assert cfg.layers[0].mixer.rot.factor is None and cfg.layers[0].mixer.chunk is None
    assert cfg.layers[3].mixer.rot is None and cfg.layers[1].ff is None and cfg.layers[2].ff is None
    names = {r.checkpoint_name for r in Model(build_topapel_spec(cfg)).weight_requests()}
    assert not names & {"l1.mlp.up", "l1.norm2", "l2.norm2"} and "l0.norm2" in names


@pytest.mark.parametrize("change,message", [
    (lambda d: d["layers"][0].__setitem__("type", "other"), "not supported"),
    (lambda d: d["layers"][0]["mixer"].__setitem__("kv_heads", 3), "multiple"),
    (lambda d: d["layers"][0]["mixer"].__setitem__("vdim", 16), "values are the keys"),
    (lambda d: d["layers"][0]["mixer"]["rot"].__setitem__("dims", 34), "fit"),
    (lambda d: d["layers"][0]["mixer"]["rot"].__setitem__("dims", 7), "even"),
    (lambda d: d["layers"][0]["mixer"]["rot"]["scaling"].__setitem__("factor", 0.0), "positive"),
    (lambda d: d["layers"][0]["mixer"]["mask"].__setitem__("size", 0), "positive"),
    (lambda d: d["layers"][0]["mixer"].pop("scale"), "lacks"),
    (lambda d: d["layers"][2]["mixer"]["decay"].append(0.5), "decay"),
    (lambda d: d["layers"][2]["mixer"]["decay"].__setitem__(0, 0.0), "decay"),
    (lambda d: d["layers"][2]["mixer"]["decay"].__setitem__(0, 1.5), "decay"),
    (lambda d: d["layers"][1]["mixer"].__setitem__("width", 0), "positive"),
    (lambda d: d["layers"][0]["mlp"].__setitem__("kind", "other"), "not supported"),
    (lambda d: d["layers"][0]["mlp"].pop("ff"), "lacks"),
    (lambda d: d.__setitem__("logit_softcap", 0.0), "logit_softcap"),
    (lambda d: d.pop("embedding"), "lacks"),
])
def test_config_errors(change, message):
    d = copy.deepcopy(tm.TA.to_hf_dict())
    change(d)
    with pytest.raises(ConfigError, match=message):
        TopapelConfig.from_hf_dict(d)


def test_tensor_names_cache_and_state():
    spec = build_topapel_spec(tm.TA)
    model = Model(spec)
    reqs = {r.checkpoint_name: r for r in model.weight_requests() if not r.alias_only}
    names = {n: r.shape for n, r in reqs.items()}
    assert names["embed"] == (150, 64) and names["final.norm"] == (64,) and "head" not in names
    assert names["l0.mix.q"] == (128, 64) and names["l0.mix.k"] == (64, 64) and "l0.mix.v" not in names
    assert names["l0.mix.q.b"] == (128,) and names["l0.mix.k.b"] == (64,) and names["l0.mix.o.b"] == (64,)
    assert names["l0.mix.q.norm"] == (32,) and names["l0.mix.k.norm"] == (32,) and names["l0.mix.sink"] == (4,)
    assert names["l0.mix.o"] == (64, 128) and names["l0.mlp.up"] == (96, 64) and names["l0.mlp.act"] == (4,)
    assert names["l1.mix.z"] == (80, 64) and names["l1.mix.x.b"] == (80,) and names["l1.mix.o"] == (64, 80)
    assert names["l2.mix.q"] == (72, 64) and names["l2.mix.v"] == (120, 64) and names["l2.mix.norm"] == (120,)
    assert names["l2.mix.g"] == (120, 64) and names["l2.mix.o"] == (64, 120) and "l2.norm2" not in names
    creq, sreq = model.cache_requests(), model.state_requests()
    assert [None if c is None else c.retention for c in creq] == [Chunks(10), None, None, Chunks(5)]
    assert [t.shape for t in creq[0].tensors] == [(2, 32), (2, 32)] and [t.shape for t in creq[3].tensors] == [(1, 32)] * 2
    assert sreq[0] is None and sreq[1].shape == (80,) and sreq[2].dtype == torch.float32 and sreq[3] is None
    assert group_windows(creq) == [Chunks(5), Chunks(10)]
    assert group_windows(Model(build_topapel_spec(tm.TB)).cache_requests()) == [None, Chunks(16)]
    assert group_windows(Model(build_topapel_spec(tm.TE)).cache_requests()) == []
    # norm weights are stored around zero: random models draw them there
    assert reqs["l0.norm1"].init.startswith("normal") and reqs["final.norm"].init.startswith("normal")


def test_parts_refuse_what_they_do_not_compute():
    base = dict(hidden_size=32, num_heads=2, num_kv_heads=1, dim=16, vdim=16, scale=0.2, eps=1e-5)
    att = get_part("mixer", "qk_norm_attention")
    with pytest.raises(ValueError, match="window or a chunk"):
        att(**base, window=4, chunk=4)
    with pytest.raises(ValueError, match="keys' size"):
        att(**dict(base, vdim=8), values="keys")
    with pytest.raises(ValueError, match="keys' size"):
        att(**base, values="keys", v_blend="source")
    with pytest.raises(ValueError, match="window or a chunk"):
        TokenCacheRequest((), window=3, chunk=3)
    with pytest.raises(ValueError, match="decay"):
        get_part("mixer", "decayed_linear_attention")(32, 2, 8, 8, (0.5,), 1e-5)
    # an arrangement that does not add a mixer's output bias refuses such a mixer
    spec = build_topapel_spec(tm.TA)
    ls = spec.layers[0]
    parallel = type(ls)(parts={"mixer": ls.parts["mixer"], "norm": PartSpec("rmsnorm", {"size": 64, "eps": 1e-5})},
                        weights={}, arrangement="parallel_residual")
    with pytest.raises(ValueError, match="output bias"):
        Model(type(spec)(**{**spec.__dict__, "layers": [parallel], "run_order": spec.run_order[:1]}))


def test_random_model_from_the_command_line(tmp_path):
    """`random-model` writes a folder for the named shape, which the plain model can run."""
    from serve_amd.__main__ import main
    folder = str(tmp_path / "a")
    assert main(["random-model", "--shape", "topapel-tiny", "--out", folder, "--seed", "5"]) == 0
    cfg = tm.plain_config(folder)
    assert TopapelConfig.from_hf_dict(cfg).to_hf_dict() == cfg
    logits = tm.plain_logits(folder, [1, 2, 3, 4, 5])
    assert logits.shape == (5, 512) and torch.isfinite(logits).all() and logits.abs().max() <= cfg["logit_softcap"]


# -- retention by chunks --------------------------------------------------------------------------------
def test_retention_rules():
    assert [first_seen(Chunks(5), p) for p in (0, 4, 5, 9, 10, 23)] == [0, 0, 5, 5, 10, 20]
    assert [first_seen(Chunks(1), p) for p in (0, 1, 7)] == [0, 1, 7]
    assert [first_seen(3, p) for p in (0, 2, 3, 9)] == [0, 0, 1, 7] and first_seen(None, 9) == 0
    assert reach(None) is None and reach(7) == 7 and reach(Chunks(7)) == 7
    assert mean_seen(Chunks(9), 1000.0) == 5.0 and mean_seen(8, 1000.0) == 8 and mean_seen(None, 10.0) == 10.0
    # the keys that tokens see, counted one by one
    for before, n in ((0, 1), (0, 23), (7, 11), (9, 1), (10, 10)):
        assert keys_seen(n, before, None, 10) == sum(p - first_seen(Chunks(10), p) + 1 for p in range(before, before + n))
        assert keys_seen(n, before, 4) == sum(p - first_seen(4, p) + 1 for p in range(before, before + n))
        assert keys_seen(n, before) == sum(p + 1 for p in range(before, before + n))


@pytest.mark.parametrize("size", [1, 3, 4, 6, 8, 13])
def test_pages_go_back_when_the_chunk_has_passed(size):
    """Page size 4; after every step the pages that are held are exactly those from the next token's chunk on (a page that
    two chunks share stays as long as the later one needs it), and never more than `max_pages_for` says."""
    cm = CacheManager([None, Chunks(size)], [64, 64], 4, 4, 64)
    for portion in (1, 2, 5, 9):
        assert cm.admit("r") is not None
        most, n = 0, 0
        while n < 60:
            n += portion
            assert cm.ensure("r", n)
            most = max(most, sum(p != FREED for p in cm.block_table("r", 1)))
            cm.trim("r", n)
            cm.check_invariants()
            first = (n // size) * size // 4
            table = cm.block_table("r", 1)
            assert [p == FREED for p in table] == [i < first for i in range(len(table))]
            assert all(p != FREED for p in cm.block_table("r", 0))
        assert most <= cm.max_pages_for(n, portion)[1] <= -(-n // 4)
        cm.release("r")
        cm.check_invariants()


def test_a_chunk_must_be_positive():
    with pytest.raises(ValueError):
        CacheManager([Chunks(0)], [4], 4, 1, 4)


# -- the plain implementation -----------------------------------------------------------------------------
def test_divided_rotation_frequencies():
    f = tp.rotary_frequencies(8, 16.0, {"factor": 4.0})
    assert torch.allclose(f, torch.tensor([0.25, 0.125, 0.0625, 0.03125], dtype=F64))
    assert torch.allclose(tp.rotary_frequencies(8, 16.0, None), 4.0 * f)
    got = rope_inverse_frequencies(8, 16.0, {"rope_type": "linear", "factor": 4.0})
    assert got.dtype == torch.float32 and torch.allclose(got.double(), f, rtol=1e-7)
    with pytest.raises(ValueError, match="not supported"):
        rope_inverse_frequencies(8, 16.0, {"rope_type": "other", "factor": 4.0})


def test_plain_rotation_and_norms():
    f = tp.rotary_frequencies(4, 10.0, {"factor": 2.0})
    x = torch.tensor([[[1.0, 2.0, 3.0, 4.0, 5.0]]], dtype=F64)
    y = tp.rotate(x, torch.tensor([3]), f)[0, 0]
    c0, s0, c1, s1 = math.cos(1.5), math.sin(1.5), math.cos(1.5 / 10 ** 0.5), math.sin(1.5 / 10 ** 0.5)
    assert torch.allclose(y, torch.tensor([1 * c0 - 3 * s0, 2 * c1 - 4 * s1, 3 * c0 + 1 * s0, 4 * c1 + 2 * s1, 5.0], dtype=F64))
    z = torch.tensor([[3.0, -4.0]], dtype=F64)
    assert torch.allclose(tp.over_rms(z, 0.0), z / math.sqrt(12.5))
    assert torch.allclose(tp.over_rms(z, 12.5), z / 5.0)
    assert torch.allclose(tp.stream_norm(z, torch.tensor([0.0, 1.0], dtype=F64), 12.5), torch.tensor([[0.6, -1.6]], dtype=F64))


def test_plain_softmax_with_sink_and_chunks():
    zero, ln2 = torch.tensor(0.0, dtype=F64), torch.tensor(math.log(2.0), dtype=F64)
    seen = tp.seen_keys(5, 2)
    assert seen.long().tolist() == [[1, 0, 0, 0, 0], [1, 1, 0, 0, 0], [0, 0, 1, 0, 0], [0, 0, 1, 1, 0], [0, 0, 0, 0, 1]]
    assert torch.equal(tp.seen_keys(4, None), torch.ones(4, 4, dtype=torch.bool).tril())
    assert torch.equal(tp.seen_keys(4, 1), torch.eye(4, dtype=torch.bool))
    s = torch.zeros(5, 5, dtype=F64)
    assert torch.allclose(tp.sink_softmax(s, seen, zero).sum(-1), torch.tensor([1 / 2, 2 / 3, 1 / 2, 2 / 3, 1 / 2], dtype=F64))
    assert torch.allclose(tp.sink_softmax(s, seen, ln2)[1], torch.tensor([1 / 4, 1 / 4, 0, 0, 0], dtype=F64))
    assert torch.allclose(tp.sink_softmax(s + 400.0, seen, ln2)[1], torch.tensor([1 / 2, 1 / 2, 0, 0, 0], dtype=F64))


def test_plain_recurrences_and_feed_forward():
    q = torch.tensor([[[1.0]], [[2.0]], [[3.0]]], dtype=F64)
    k = torch.tensor([[[1.0]], [[10.0]], [[100.0]]], dtype=F64)
    v = torch.ones(3, 1, 1, dtype=F64)
    o = tp.decayed_outer_products(q, k, v, torch.tensor([0.5], dtype=F64))[:, 0, 0]
    assert o.tolist() == [1.0, 2 * 10.5, 3 * 105.25]
    g = torch.Generator().manual_seed(0)
    q, k, v = (torch.randn(4, 2, 3, generator=g, dtype=F64) for _ in range(3))
    a = torch.tensor([0.7, 1.0], dtype=F64)
    want = torch.zeros_like(v)
    for t in range(4):
        for s in range(t + 1):
            want[t] += (a ** (t - s))[:, None] * (q[t] * k[s]).sum(-1, keepdim=True) * v[s]
    assert torch.allclose(tp.decayed_outer_products(q, k, v, a), want)
    u = torch.tensor([-2.0, 0.0, 3.0], dtype=F64)
    assert torch.allclose(tp.positive_part(u), torch.tensor([1 / (1 + math.exp(2.0)), 0.5, 3.5], dtype=F64))
    z = torch.tensor([[0.25], [0.5], [1.0]], dtype=F64)
    c = torch.tensor([[4.0], [2.0], [7.0]], dtype=F64)
    assert tp.gated_average(z, c)[:, 0].tolist() == [1.0, 1.5, 7.0]
    y = torch.tensor([[1.0, -2.0]], dtype=F64)
    coef = torch.tensor([2.0, 3.0, 5.0, 7.0], dtype=F64)
    r1, r2, r3 = math.sqrt(2.5), math.sqrt(8.5), math.sqrt(32.5)
    want = torch.tensor([[2 / r1 + 3 / r2 + 5 / r3 + 7, -4 / r1 + 12 / r2 - 40 / r3 + 7]], dtype=F64)
    assert torch.allclose(tp.poly_norm(y, coef, 0.0), want)
    assert tp.soft_cap(torch.tensor(4.0, dtype=F64), 2.0).item() == pytest.approx(2.0 * math.tanh(2.0))


def test_every_mechanism_shows_in_the_plain_logits(tmp_path):
    """Leaving a mechanism out, or moving an edge by one, moves the plain model's logits by 150 times the float32
    tolerance and more (chunks, values, sinks, states and decays by more than the bfloat16 tolerance): a fault of that
    kind in the engine cannot hide behind the tolerances."""
    folder = tm.make_folder(tmp_path, "TAsharp", config=tm.TA, seed=3, scales=tm.SHARP)
    cfg, weights = tm.plain_config(folder), tm.plain_weights(folder)
    tokens = [(7 * i * i + 3 * i + 1) % 150 for i in range(44)]
    want = tm.plain_logits(folder, tokens)

    def moved(config=None, tensors=None, fn=None):
        if fn is not None:
            saved = {n: getattr(tp, n) for n in fn}
            for n, f in fn.items():
                setattr(tp, n, f)
        try:
            got = tm.plain_logits(folder, tokens, config, tensors)
        finally:
            if fn is not None:
                for n, f in saved.items():
                    setattr(tp, n, f)
        return tm.row_distance(got, want)[-14:].max().item()

    exact, coarse = 150 * tm.TOLERANCE["float32"], 1.2 * tm.TOLERANCE["bfloat16"]

    def edit(*path_and_value):
        c = copy.deepcopy(cfg)
        at = c
        for key in path_and_value[:-2]:
            at = at[key]
        at[path_and_value[-2]] = path_and_value[-1]
        return c
    for layer, size in ((0, 9), (0, 11), (3, 4), (3, 6)):
        assert moved(edit("layers", layer, "mixer", "mask", "size", size)) > coarse, f"chunks of layer {layer} at {size}"
    assert moved(edit("layers", 0, "mixer", "rot", "scaling", None)) > exact
    assert moved(edit("layers", 2, "mixer", "decay", [0.5, 0.9, 1.0])) > exact
    assert moved(edit("layers", 2, "mixer", "decay", [0.5, 0.95, 0.99])) > exact
    assert moved(edit("logit_scale", 1.0)) > exact
    assert moved(edit("logit_softcap", 60.0)) > exact
    assert moved(edit("embedding", "scale", 1.0)) > exact
    for name in ("l0.mix.q.b", "l0.mix.k.b", "l0.mix.o.b", "l3.mix.o.b", "l0.mix.q.norm", "l0.mix.k.norm", "l1.mix.z.b", "l1.mix.x.b",
                 "l1.mix.g", "l2.mix.g", "l2.mix.norm", "l0.norm1", "l1.norm2", "final.norm"):
        w = dict(weights)
        w[name] = torch.ones_like(w[name]) if name.endswith(("q.norm", "k.norm", "mix.norm")) else torch.zeros_like(w[name])
        assert moved(tensors=w) > exact, name
    for i in range(4):
        w = dict(weights)
        w["l0.mlp.act"] = w["l0.mlp.act"].clone()
        w["l0.mlp.act"][i] = 0.0
        assert moved(tensors=w) > exact, f"term {i} of the activation"
    soft, gated, outer = tp.sink_softmax, tp.gated_average, tp.decayed_outer_products
    assert moved(fn={"sink_softmax": lambda s, seen, sink: soft(s, seen, torch.tensor(-1e9, dtype=F64))}) > coarse     # no sink
    assert moved(fn={"sink_softmax": lambda s, seen, sink: soft(s, seen, 0.3 * sink)}) > exact               # a scaled sink
    assert moved(fn={"rotate": lambda x, p, f: x}) > coarse
    # a state that is lost after 30 tokens
    assert moved(fn={"gated_average": lambda z, c: torch.cat([gated(z[:30], c[:30]), gated(z[30:], c[30:])])}) > exact
    assert moved(fn={"decayed_outer_products": lambda q, k, v, a: torch.cat(
        [outer(q[:30], k[:30], v[:30], a), outer(q[30:], k[30:], v[30:], a)])}) > coarse
    assert moved(fn={"positive_part": lambda u: u}) > exact

    def normed_values(h, t, p, m, eps):                     # (the values behind the norm instead of in front of it)
        T, H, G, D = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
        q = tp.over_rms((h @ t[p + "q"].T + t[p + "q.b"]).view(T, H, D), eps) * t[p + "q.norm"]
        k = tp.over_rms((h @ t[p + "k"].T + t[p + "k.b"]).view(T, G, D), eps) * t[p + "k.norm"]
        f = tp.rotary_frequencies(m["rot"]["dims"], m["rot"]["base"], m["rot"].get("scaling"))
        qr, kr = tp.rotate(q, torch.arange(T), f), tp.rotate(k, torch.arange(T), f)
        seen = tp.seen_keys(T, m["mask"]["size"])
        out = [tp.sink_softmax(qr[:, i] @ kr[:, i // (H // G)].T * m["scale"], seen, t[p + "sink"][i]) @ k[:, i // (H // G)]
               for i in range(H)]
        return torch.cat(out, -1) @ t[p + "o"].T + t[p + "o.b"]
    assert moved(fn={"attention_mixer": normed_values}) > coarse
