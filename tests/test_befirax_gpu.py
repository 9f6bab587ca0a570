"""The Befirax decoder through the engine against the plain implementation, float32 and bfloat16: whole prompts and
first tokens; prompt then token by token; portions down to two tokens; unequal requests in one batch against each
alone, with pages and slots that are freed and used again; windows' edges with sharp scores, in prompts and in decoding;
a far key among hundreds, at page borders, also through a layer that reads another's keys; long prompts and long
decoding; greedy generation through the scheduler; the trace runner as a program; and the kernels alone."""
from __future__ import annotations

import dataclasses
import os
import random
from types import SimpleNamespace

import pytest
import torch

from tests import befirax_models as bm
from tests.plain import befirax_plain as bp

pytestmark = pytest.mark.gpu

DTYPES = ["float32", "bfloat16"]
NAMES = list(bm.MODELS)
F64 = torch.float64


def tokens_for(n, seed, vocab):
    rng = random.Random(seed)
    return [rng.randrange(vocab) for _ in range(n)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_whole_prompts_and_first_tokens(tmp_path, name, dtype):
    folder = bm.make_folder(tmp_path, name)
    engine = bm.engine_for(folder, dtype)
    vocab = bm.MODELS[name][0].vocab
    for n in (1, 2, 3, 5, 61, 131):
        tokens = tokens_for(n, 100 + n, vocab)
        got = bm.run_portions(engine, f"r{n}", tokens, [n])
        bm.assert_matches_plain(got, folder, tokens, dtype, f"{name} whole {n}")
    engine.runner.cache.check_invariants()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_prompt_then_token_by_token(tmp_path, name, dtype):
    folder = bm.make_folder(tmp_path, name)
    engine = bm.engine_for(folder, dtype)
    vocab = bm.MODELS[name][0].vocab
    tokens = tokens_for(84, 7, vocab)
    got = bm.run_portions(engine, "r", tokens, [84 - 45] + [1] * 45)
    bm.assert_matches_plain(got, folder, tokens, dtype, f"{name} prompt + 45 single tokens")
    got = bm.run_portions(engine, "s", tokens[:30], [1] * 30)             # from the very first token on
    bm.assert_matches_plain(got, folder, tokens[:30], dtype, f"{name} token by token from the start")
    if dtype == "float32":
        whole = bm.run_portions(engine, "w", tokens, [84])
        assert bm.row_distance(got, whole[:30]).max().item() <= 3e-5


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_portions_of_changing_size(tmp_path, name, dtype):
    folder = bm.make_folder(tmp_path, name)
    engine = bm.engine_for(folder, dtype)
    vocab = bm.MODELS[name][0].vocab
    tokens = tokens_for(173, 8, vocab)
    for portions in ([7, 2, 16, 3, 2, 9, 2, 11, 5, 4, 1, 1, 2, 8, 100], [2] * 10 + [53, 17, 83], [1, 3, 169], [40, 33, 32, 68]):
        got = bm.run_portions(engine, "r", tokens, portions)
        bm.assert_matches_plain(got, folder, tokens, dtype, f"{name} portions {portions}")


# BA without its routers: no row rests on a close call, so that bfloat16 rows are all compared
BA_ATTENTION = dataclasses.replace(bm.BA, layers=tuple(dataclasses.replace(l, mlp=None) for l in bm.BA.layers))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("page_size", [4, 16])
def test_windows_edges_with_sharp_scores(tmp_path, dtype, page_size):
    """Scores drawn wider, so that a key just inside or just outside a window (10 and 5 positions; a page holds 4 or 16)
    carries weight.  Portions that end before, at and behind multiples of the windows, and single tokens across many of
    them; pages that no later token sees go back to the pool on the way and are NaN until written again."""
    folder = bm.make_folder(tmp_path, "BAwindows", config=BA_ATTENTION, seed=3, scales=bm.EDGES)
    engine = bm.engine_for(folder, dtype, num_pages=192 // page_size, page_size=page_size, debug_poison_cache=True)
    tokens = tokens_for(90, 21, bm.BA.vocab)
    want = bm.plain_logits(folder, tokens)
    for layer, sizes in ((1, (9, 11)), (4, (4, 6))):
        for size in sizes:                  # (a window one off would show in many rows)
            c = bm.plain_config(folder)
            c["layers"][layer]["mixer"]["mask"]["size"] = size
            assert bm.row_distance(bm.plain_logits(folder, tokens, c), want).median().item() > 100 * bm.TOLERANCE["float32"]
    for portions in ([90], [4, 1, 5, 1, 9, 10, 11, 2, 3] + [1] * 44, [9, 2] + [1] * 30 + [49], [5] * 18, [10] * 9):
        got = bm.run_portions(engine, "r", tokens, portions)
        bm.assert_matches_plain(got, folder, tokens, dtype, f"sharp windows, portions {portions[:9]}...")
    engine.runner.cache.check_invariants()


def mixed_trace(rng, reqs, max_live=4):
    """Up to `max_live` live requests; portions of some beside single tokens of others; staggered."""
    fed = {k: 0 for k in reqs}
    order, live, steps, nxt = list(reqs), [], [], 0
    while nxt < len(order) or live:
        while len(live) < max_live and nxt < len(order) and (not live or rng.random() < 0.6):
            live.append(order[nxt])
            nxt += 1
        entries, ended = [], []
        for k in list(live):
            if rng.random() < 0.2 and len(live) > 1:
                continue                         # left out of this step, goes on later
            n = min(len(reqs[k]) - fed[k], rng.choice([1, 1, 1, 2, 3, 5, 8, 13, 40]))
            entries.append((k, reqs[k][fed[k]: fed[k] + n]))
            fed[k] += n
            if fed[k] == len(reqs[k]):
                ended.append(k)
                live.remove(k)
        if entries:
            steps.append((entries, ended))
    return steps


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_unequal_requests_together_with_pages_and_slots_used_again(tmp_path, name, dtype):
    from serve_amd.engine.batch import Segment
    folder = bm.make_folder(tmp_path, name)
    lengths = [23, 71, 9, 30, 117, 2, 36, 1, 60, 28, 33, 5]
    # four live requests: pool and slots are far fewer than the requests need together
    engine = bm.engine_for(folder, dtype, num_pages=71, page_size=4, max_requests=4, debug_poison_cache=True)
    vocab = bm.MODELS[name][0].vocab
    reqs = {f"q{i}": tokens_for(n, 300 + i, vocab) for i, n in enumerate(lengths)}
    steps = mixed_trace(random.Random(13), reqs)
    rows = {k: [] for k in reqs}
    slots_seen, pages_seen = {}, {}
    for entries, ended in steps:
        segs = []
        for k, toks in entries:
            if k not in engine.runner.cache:
                assert engine.runner.admit(k)
                slots_seen.setdefault(engine.runner.cache.slot_of(k), []).append(k)
            segs.append(Segment(k, toks, list(range(len(toks)))))
        logits = engine.step(segs)
        at = 0
        for k, toks in entries:
            rows[k].append(logits[at: at + len(toks)])
            at += len(toks)
            for page in engine.runner.cache.block_table(k, 0):
                pages_seen.setdefault(page, set()).add(k)
        for k in ended:
            engine.runner.release(k)
    engine.runner.cache.check_invariants()
    assert max(len(v) for v in slots_seen.values()) >= 3 and max(len(v) for v in pages_seen.values()) >= 3
    for k, toks in reqs.items():
        bm.assert_matches_plain(torch.cat(rows[k]), folder, toks, dtype, f"{name} request {k} in the mix")


def far_key_model(tmp_path, n, far):
    """Attention alone, on one layer's keys, and an embedding table made so that one score stands out: token 1's row is
    set so that its first maps' queries point along the first map's key of token 0 at position `far`, as rotated to
    position n - 1, and its second maps' queries are nothing.  A sequence that ends in token 1 and holds token 0 once, at
    `far`, then reads that key with nearly all of its first map's weight.  Queries and keys pass the convolution unchanged."""
    from safetensors.torch import save_file
    rot = bm.ROT(1000.0, 8)
    cfg = bm.BefiraxConfig(vocab=90, width=128, eps=1e-5, streams=3, layers=(
        bm.L(bm.ATT(2, 1, 16, 24, 3.0, 0.2, 3, rot), None),))
    folder = bm.make_folder(tmp_path, f"far{far}", config=cfg, seed=11, scales={r"q\.b$": 0.0})
    out = bm.plain_weights(folder)
    for name in ("l0.mix.q.conv", "l0.mix.k.conv"):
        out[name].zero_()
        out[name][:, -1] = 1
    W = {k: v.double() for k, v in out.items()}
    a = W["l0.hc1.in"].sum()
    h0 = bp.rms_norm(a * W["embed"][0:1], W["l0.norm1"], 1e-5)
    k0 = (h0 @ W["l0.mix.k"].T + W["l0.mix.k.b"])[0, :16]                     # the first map's key
    turned = bp.rotate(torch.stack([k0] * (n + 1)), 8, 1000.0, "interleaved")
    # the query that, turned to n - 1, lies along the key as turned to `far`: turned back by the distance
    back = k0.clone()
    f = 1000.0 ** (-2.0 * torch.arange(4, dtype=F64) / 8)
    ang = (far - (n - 1)) * f
    back[0:8:2], back[1:8:2] = (k0[0:8:2] * ang.cos() - k0[1:8:2] * ang.sin(), k0[1:8:2] * ang.cos() + k0[0:8:2] * ang.sin())
    assert torch.allclose(bp.rotate(torch.stack([back] * n), 8, 1000.0, "interleaved")[n - 1], turned[far], atol=1e-9)
    target = torch.cat([back, torch.zeros(16, dtype=F64)] * 2)
    row = (torch.linalg.pinv(W["l0.mix.q"]) @ target) / W["l0.norm1"]
    out["embed"][1] = (0.28 * row / row.pow(2).mean().sqrt()).to(out["embed"].dtype)      # (as large as the other rows)
    save_file({k: v.contiguous() for k, v in out.items()}, os.path.join(folder, "model.safetensors"))
    return folder


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_far_key_among_hundreds(tmp_path, dtype):
    rng = random.Random(5)
    n = 420
    for far in (3, 37, 203):                  # in the first page, further on, and the last key of a page (page size 4)
        folder = far_key_model(tmp_path, n, far)
        with_key = [rng.randrange(2, 90) for _ in range(n - 1)] + [1]
        with_key[far] = 0
        without = list(with_key)
        without[far] = 2
        want = bm.plain_logits(folder, with_key)[-1:]
        # losing that one key would move the last row by far more than the tolerance
        assert bm.row_distance(bm.plain_logits(folder, without)[-1:], want).item() > 2 * bm.TOLERANCE["bfloat16"]
        engine = bm.engine_for(folder, dtype, num_pages=120, page_size=4)
        got = bm.run_portions(engine, "r", with_key, [n - 3, 1, 1, 1])[-1:]
        bm.assert_rows_close(got, want, dtype, f"key {far} of {n}, read by a token decoded alone")
        got = bm.run_portions(engine, "r", with_key, [200, 220])[-1:]
        bm.assert_rows_close(got, want, dtype, f"key {far} of {n}, read from a portion")


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_shared_cache_over_hundreds_of_keys_with_sharp_scores(tmp_path, dtype):
    """BF's three layers all read the first one's keys: drawn wide, every query puts its weight on a few keys anywhere
    in the 300 tokens before it, so keys lost far back, or at a page's border, would show in many rows."""
    cfg = dataclasses.replace(bm.BF, layers=tuple(dataclasses.replace(l, mlp=None) for l in bm.BF.layers))
    folder = bm.make_folder(tmp_path, "BFsharp", config=cfg, seed=17, scales={r"mix\.(q|k)$": 2.5})
    tokens = tokens_for(300, 41, cfg.vocab)
    want = bm.plain_logits(folder, tokens)
    soft = bp.softmax_weights
    try:                                        # (what losing the keys more than 100 back would do to the last rows)
        bp.softmax_weights = lambda s, window: soft(s, 100)
        short = bm.plain_logits(folder, tokens)
    finally:
        bp.softmax_weights = soft
    assert bm.row_distance(short[-50:], want[-50:]).median().item() > 2 * bm.TOLERANCE["bfloat16"]
    engine = bm.engine_for(folder, dtype, num_pages=90, page_size=4)
    got = bm.run_portions(engine, "r", tokens, [250] + [1] * 30 + [20])
    bm.assert_matches_plain(got, folder, tokens, dtype, "sharp differential attention over 300 keys")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["BB", "BF"])
def test_long_prompts(tmp_path, name, dtype):
    """Prompts long enough for the kernels that take runs of tokens, whole and behind a first portion that leaves the
    runs across the pages' borders."""
    folder = bm.make_folder(tmp_path, name)
    engine = bm.engine_for(folder, dtype, num_pages=100)
    tokens = tokens_for(701, 23, bm.MODELS[name][0].vocab)
    for portions in ([701], [3, 698]):
        got = bm.run_portions(engine, "r", tokens, portions)
        bm.assert_matches_plain(got, folder, tokens, dtype, f"{name} {portions}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["BA", "BB"])
def test_long_decoding(tmp_path, name, dtype):
    folder = bm.make_folder(tmp_path, name)
    engine = bm.engine_for(folder, dtype, num_pages=80)
    vocab = bm.MODELS[name][0].vocab
    tokens = tokens_for(260, 31, vocab)
    got = bm.run_portions(engine, "r", tokens, [4] + [1] * 256)
    bm.assert_matches_plain(got, folder, tokens, dtype, f"{name} 256 single tokens")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["BA", "BC"])
def test_greedy_generation_through_the_scheduler(tmp_path, name, dtype):
    """`generate` (scheduler, mixed steps, graphs, steps launched ahead of the host) picks the tokens the plain model
    picks, as long as the plain model's choice is clear."""
    from serve_amd.engine.engine import Request
    folder = bm.make_folder(tmp_path, name)
    engine = bm.engine_for(folder, dtype, num_pages=128, page_size=8, max_requests=3)
    vocab = bm.MODELS[name][0].vocab
    prompts = [tokens_for(n, 50 + n, vocab) for n in (5, 19, 1, 33, 8)]
    new = 12
    reqs = [Request(torch.tensor(p), len(p), new) for p in prompts]
    out = engine.generate(reqs, temperature=0.0, return_logits="all")
    compared = 0
    for p, o in zip(prompts, out):
        assert o.error is None and len(o.generated_tokens) == new
        seq = list(p)
        for i, tok in enumerate(o.generated_tokens.tolist()):
            row = bm.plain_logits(folder, seq)[-1]
            top2 = row.topk(2).values
            if (top2[0] - top2[1]).item() < (1e-3 if dtype == "float32" else 0.15) * row.std().item():
                break                            # the plain model's own choice is a close call: stop comparing
            assert tok == int(row.argmax()), f"{name}: token {i} after a prompt of {len(p)}"
            if dtype == "float32":
                bm.assert_rows_close(o.logits[i: i + 1], row[None], dtype, f"{name} logits of generated token {i}")
            seq.append(tok)
            compared += 1
    assert compared >= (new if dtype == "float32" else 5)
    engine.runner.cache.check_invariants()
    assert engine.runner.cache.free_slots() == 3
    # without the logits the scheduler samples on the device and replays decode steps from graphs: the same tokens
    again = engine.generate([Request(torch.tensor(p), len(p), new) for p in prompts], temperature=0.0)
    if dtype == "float32":
        assert [o.generated_tokens.tolist() for o in again] == [o.generated_tokens.tolist() for o in out]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["BA", "BD"])
def test_steps_replayed_from_graphs_give_the_eager_logits(tmp_path, name, dtype):
    """Two requests decoded side by side, eagerly and through a captured graph that is replayed many times."""
    from serve_amd.engine.batch import Segment
    folder = bm.make_folder(tmp_path, name)
    vocab = bm.MODELS[name][0].vocab
    a, b = tokens_for(40, 1, vocab), tokens_for(33, 2, vocab)
    rows = {}
    for graphs in (False, True):
        engine = bm.engine_for(folder, dtype, use_graphs=graphs)
        for k, t in (("a", a), ("b", b)):
            assert engine.runner.admit(k)
            engine.step([Segment(k, t[:9], [])])
        out = [engine.step([Segment("a", [a[9 + i]], [0]), Segment("b", [b[9 + i]], [0])]) for i in range(24)]
        rows[graphs] = torch.stack(out).cpu()
    assert bm.row_distance(rows[True].view(48, -1), rows[False].view(48, -1)).max().item() <= (3e-5 if dtype == "float32" else 2e-2)


@pytest.mark.parametrize("dtype", DTYPES)
def test_traces_through_the_program(tmp_path, dtype):
    """`bin/trace_run` as a child process on a model folder: whole prompts, prompt then single tokens, portions, and a
    mix of four live requests (four state slots, pages for 256 tokens), against the plain model."""
    import json
    import subprocess
    import numpy as np
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    name = "BA"
    folder = bm.make_folder(tmp_path, name)
    vocab = bm.MODELS[name][0].vocab
    reqs, steps = {}, []

    def feed(key, n, portions, seed):
        reqs[key] = tokens_for(n, seed, vocab)
        at = 0
        for j, m in enumerate(portions):
            steps.append(([(key, reqs[key][at: at + m])], [key] if j == len(portions) - 1 else []))
            at += m
        assert at == n
    feed("whole", 50, [50], 1)
    feed("tail", 70, [30] + [1] * 40, 2)
    feed("cut", 61, [7, 2, 16, 3, 2, 9, 2, 11, 5, 4], 3)
    mixed = {f"m{i}": tokens_for(n, 40 + i, vocab) for i, n in enumerate([23, 41, 9, 30, 17, 2, 36, 12, 40])}
    reqs.update(mixed)
    steps.extend(mixed_trace(random.Random(5), mixed))
    lines = [json.dumps({"step": i, "entries": [{"id": k, "tokens": t, "want": list(range(len(t)))} for k, t in entries],
                         "end": ended}) for i, (entries, ended) in enumerate(steps)]
    out = tmp_path / "out"
    proc = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", dtype, "--out", str(out),
                           "--max-tokens", "256"], input="\n".join(lines) + "\n", capture_output=True, text=True, timeout=600)
    assert proc.returncode == 0, proc.stderr[-3000:]
    assert [l for l in proc.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(len(steps))]
    rows = {k: [] for k in reqs}
    for i, (entries, _) in enumerate(steps):
        arr = torch.from_numpy(np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(sum(len(t) for _, t in entries), vocab))
        at = 0
        for k, t in entries:
            rows[k].append(arr[at: at + len(t)])
            at += len(t)
    assert sum(len(t) for t in reqs.values()) > 256          # pages went from request to request
    for k, t in reqs.items():
        bm.assert_matches_plain(torch.cat(rows[k]), folder, t, dtype, f"trace request {k}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_checkpoint_with_tensors_in_32_bit(tmp_path, dtype):
    """Gates, corrections, norms and stream weights stored in float32 keep their precision in the bfloat16 engine (and
    the products that put several matrices together are then made apart, or in float32)."""
    from safetensors.torch import save_file
    folder = bm.make_folder(tmp_path, "BA32", config=bm.BA, seed=3)
    g = torch.Generator().manual_seed(1)
    out = {}
    for name, t in bm.plain_weights(folder).items():
        if name.endswith((".g", ".correction", ".in", ".out", ".mix", ".norm1", ".norm2", ".b", ".conv")) and not name.endswith("mix.in"):
            t = t.float() * (1 + 1e-3 * torch.randn(t.shape, generator=g))
        out[name] = t.contiguous()
    save_file(out, os.path.join(folder, "model.safetensors"))
    engine = bm.engine_for(folder, dtype)
    tokens = tokens_for(70, 15, bm.BA.vocab)
    got = bm.run_portions(engine, "r", tokens, [40] + [1] * 20 + [10])
    bm.assert_matches_plain(got, folder, tokens, dtype, "tensors in 32 bit")


# ---------------------------------------------------------------------------------------------
# the kernels alone
# ---------------------------------------------------------------------------------------------
def _step(lens, slots, positions0, dev="cuda"):
    """A step's index arrays for segments of the given lengths."""
    cu = [0]
    for n in lens:
        cu.append(cu[-1] + n)
    seg = [i for i, n in enumerate(lens) for _ in range(n)]
    pos = [p + j for p, n in zip(positions0, lens) for j in range(n)]
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=dev)          # noqa: E731
    return SimpleNamespace(num_tokens=cu[-1], num_segments=len(lens), positions=i32(pos), seg_of_token=i32(seg), cu_q=i32(cu),
                           state_slots=i32(slots), max_q_len=max(lens))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("S,d,T", [(4, 64, 5), (2, 512, 300), (3, 2304, 3), (1, 50, 7), (4, 50, 6), (5, 96, 4), (16, 30, 2),
                                   (4, 4096, 2), (3, 260, 400)])
def test_stream_mix(dtype, S, d, T):
    """Every form of a sublayer's output (none, rows, partial sums, experts' rows some of which are identity experts),
    with and without a bias, all rows and some, against float64."""
    from serve_amd import ops
    g = torch.Generator().manual_seed(S * d + T)
    r = lambda *s: torch.randn(*s, generator=g)                              # noqa: E731
    X0 = r(T, S, d).cuda()
    M, b, a, w, bias = r(S, S).cuda(), r(S).cuda(), r(S).cuda(), (1 + 0.1 * r(d)).cuda(), r(d).cuda()
    own = r(T, d).to(dtype).cuda()
    forms = {"none": None, "rows": r(T, d).to(dtype).cuda(), "fp32": r(T, d).cuda()}
    for p in (1, 3, 8, 9):
        forms[f"parts{p}"] = r(p, T, d).cuda()
    for top in (1, 4, 7, 9):
        yk = r(T * top, d).cuda()
        ids = torch.randint(0, 6, (T, top), generator=g).int().cuda()
        yk[(ids >= 4).view(-1)] = float("nan")                               # an identity expert's row holds nothing
        forms[f"experts{top}"] = ops.ExpertRows(yk, r(T, top).cuda(), ids, 4, own)
    eps = 1e-5
    for name, y in forms.items():
        for use_bias in (False, True):
            X, MD = X0.double(), M.double()
            if y is not None:
                if isinstance(y, ops.ExpertRows):
                    top = y.weights.shape[1]
                    rows_ = torch.where((y.ids >= 4)[..., None], own.double()[:, None], y.yk.double().view(T, top, d))
                    yy = (rows_ * y.weights.double()[..., None]).sum(1)
                else:
                    yy = y.double().sum(0) if y.dim() == 3 else y.double()
                if use_bias:
                    yy = yy + bias.double()
                # (einsum over streams of a few numbers: written as a sum, the copies stay apart)
                X = torch.stack([sum(MD[s, t] * X[:, s] for s in range(S)) + b.double()[t] * yy for t in range(S)], dim=1)
            u = sum(a.double()[s] * X[:, s] for s in range(S))
            want = u / torch.sqrt(u.pow(2).mean(-1, keepdim=True) + eps) * w.double()
            x = X0.clone()
            out = torch.empty((T, d), dtype=dtype, device="cuda")
            args = (y, bias if use_bias else None, M, b) if y is not None else (None, None, None, None)
            ops.stream_mix(x, *args, a, w, eps, out)
            tol = dict(atol=2e-4, rtol=1e-4) if dtype == torch.float32 else dict(atol=3e-2, rtol=1e-2)
            assert torch.allclose(x.double(), X, atol=2e-4, rtol=1e-4), f"{name}: the streams"
            assert torch.allclose(out.double(), want, **tol), f"{name}: the norm"
            rows = torch.tensor([T - 1, 0, T // 2], dtype=torch.int32, device="cuda")
            x = X0.clone()
            part = torch.empty((3, d), dtype=dtype, device="cuda")
            ops.stream_mix(x, *args, a, w, eps, part, rows)
            assert torch.equal(x, X0) and torch.allclose(part.double(), want[rows.long()], **tol), f"{name}: some rows"


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,M,D,Dv,Dp,rot,adjacent,taps,long", [
    (4, 2, 2, 24, 40, 48, 8, True, 3, 0), (6, 3, 2, 16, 32, 32, 16, True, 4, 0), (3, 3, 2, 6, 7, 16, 4, True, 1, 0),
    (2, 1, 2, 72, 24, 144, 36, True, 5, 0), (4, 2, 1, 32, 16, 32, 32, False, 4, 0), (2, 1, 3, 8, 24, 32, 6, True, 2, 0),
    (6, 3, 2, 16, 32, 32, 16, True, 4, 1), (4, 2, 2, 32, 64, 64, 12, True, 2, 1), (2, 2, 2, 8, 16, 16, 0, True, 3, 1),
    (4, 1, 2, 24, 40, 48, 8, True, 1, 1), (3, 1, 2, 10, 7, 32, 4, True, 3, 1)])
def test_conv_rope_kv_write(dtype, H, G, M, D, Dv, Dp, rot, adjacent, taps, long):
    """Requests over three steps (portions of unequal length, single tokens, portions again; one without a cache slot
    or state), also long enough for runs of eight tokens across segments' and pages' borders; with slots used by an
    earlier request; queries alone; against the convolution over whole sequences."""
    from serve_amd import ops
    page = 8
    C = H * M * D + G * (M * D + Dv)
    g = torch.Generator().manual_seed(H * D + taps + long)
    lens = [[300, 5, 2, 420], [1, 1, 1, 1], [37, 600, 3, 1]] if long else [[7, 1, 2, 5], [1, 1, 1, 1], [3, 1, 6, 1]]
    total = [sum(s[i] for s in lens) for i in range(4)]
    seqs = [torch.randn(n, C, generator=g).to(dtype) for n in total]
    bias, w = torch.randn(C, generator=g), torch.randn(C, taps, generator=g)
    P = sum(-(-n // page) for n in total) + 3
    base, at = [], 1
    for n in total:                                     # (every sequence in pages of its own, the last page first)
        np_ = -(-n // page)
        base.append([at + np_ - 1 - i for i in range(np_)])
        at += np_
    slot_of = [2, 0, -1, 1]                             # (the third request is of no slot: nothing of it is kept)
    freq = (100.0 ** (-2.0 * torch.arange(max(rot // 2, 1), dtype=F64) / max(rot, 1)))[: rot // 2].float().cuda()
    for with_bias in (True, False):
        state = torch.full((3, (taps - 1) * C + 4), 7.0, device="cuda")       # (stale rows: position 0 must not read them)
        qstate = torch.full((3, (taps - 1) * H * M * D + 4), 7.0, device="cuda")
        k_pages = torch.full((P, G, page, Dp), 9.0, dtype=dtype, device="cuda")
        v_pages = torch.full((P, G, Dp, page), 9.0, dtype=dtype, device="cuda")
        b = bias if with_bias else None
        done = [0] * 4
        tol = dict(atol=2e-3, rtol=1e-4) if dtype == torch.float32 else dict(atol=6e-2, rtol=2e-2)
        full = []
        for i in range(4):
            u = seqs[i].double() + (bias.double() if with_bias else 0.0)
            if slot_of[i] < 0:
                full.append(None)
                continue
            y = bp.causal_conv(u, w.double())
            q = y[:, : H * M * D].reshape(-1, H, M, D)
            k = y[:, H * M * D: (H + G) * M * D].reshape(-1, G, M, D)
            layout = "interleaved" if adjacent else "half"
            if rot:
                q, k = bp.rotate(q, rot, 100.0, layout), bp.rotate(k, rot, 100.0, layout)
            full.append((q, k, y[:, (H + G) * M * D:].reshape(-1, G, Dv)))
        for step in lens:
            z = torch.cat([seqs[i][done[i]: done[i] + step[i]] for i in range(4)])
            z = torch.cat([z, torch.full((z.shape[0], 8 if H % 2 == 0 else 5), 3.0, dtype=dtype)], dim=1).contiguous().cuda()
            ctx = _step(step, slot_of, done)
            slots = []
            for i in range(4):
                for p in range(done[i], done[i] + step[i]):
                    slots.append(-1 if slot_of[i] < 0 else base[i][p // page] * page + p % page)
            slots = torch.tensor(slots, dtype=torch.int32, device="cuda")
            q_out = torch.full((ctx.num_tokens, H * M * Dp), 9.0, dtype=dtype, device="cuda")
            ops.conv_rope_kv_write(z, None if b is None else b.cuda(), w.cuda(), state[:, :-4], 0, ctx, q_out, slots, k_pages,
                                   v_pages, freq if rot else None, rot, adjacent, H, G, M, D, Dv)
            # the same queries where nothing is stored (a layer that reads another's keys)
            q_alone = torch.full_like(q_out, 9.0)
            cq = H * M * D
            ops.conv_rope_kv_write(z, None if b is None else b[:cq].contiguous().cuda(), w[:cq].contiguous().cuda(), qstate[:, :-4],
                                   0, ctx, q_alone, None, None, None, freq if rot else None, rot, adjacent, H, G, M, D, Dv)
            live = torch.cat([torch.full((n,), slot_of[i] >= 0) for i, n in enumerate(step)])
            assert torch.equal(q_alone.cpu()[live], q_out.cpu()[live])
            qq = q_out.double().cpu().view(-1, H, M, Dp)
            off = 0
            for i in range(4):
                if full[i] is not None:
                    want = full[i][0][done[i]: done[i] + step[i]]
                    got = qq[off: off + step[i]]
                    for m in range(M):
                        assert torch.allclose(got[:, :, m, m * D: (m + 1) * D], want[:, :, m], **tol)
                        assert (got[:, :, m, : m * D] == 0).all() and (got[:, :, m, (m + 1) * D:] == 0).all()
                off += step[i]
                done[i] += step[i]
        used = torch.zeros(P, page, dtype=torch.bool)
        for i in range(4):
            if full[i] is None:
                continue
            p = torch.arange(total[i])
            pages, offs = torch.tensor(base[i])[p // page], p % page
            used[pages, offs] = True
            kk, vv = k_pages.double().cpu()[pages, :, offs], v_pages.double().cpu()[pages, :, :, offs]
            assert torch.allclose(kk[..., : M * D], full[i][1].reshape(-1, G, M * D), **tol) and (kk[..., M * D:] == 0).all()
            assert torch.allclose(vv[..., :Dv], full[i][2], **tol) and (vv[..., Dv:] == 0).all()
            if taps > 1:
                kept = state[slot_of[i], : (taps - 1) * C].view(taps - 1, C).cpu()
                n = min(taps - 1, total[i])              # (a shorter sequence has left the oldest rows as they were)
                assert torch.equal(kept[taps - 1 - n:], seqs[i][-n:].float())
        free = (~used).nonzero()
        assert (k_pages.cpu()[free[:, 0], :, free[:, 1]] == 9).all() and (v_pages.cpu()[free[:, 0], :, :, free[:, 1]] == 9).all()
        assert (state[:, -4:] == 7).all()                # nothing behind the rows' convolution inputs is touched


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,Dv,Dp,T", [(4, 40, 48, 5), (3, 7, 16, 6), (6, 128, 128, 300), (1, 1, 16, 3), (2, 300, 304, 4),
                                       (2, 640, 640, 2), (5, 64, 96, 17)])
def test_differential_heads(dtype, H, Dv, Dp, T):
    from serve_amd import ops
    g = torch.Generator().manual_seed(H * Dv)
    a = torch.randn(T, 2 * H * Dp, generator=g).to(dtype).cuda()
    rows = torch.randn(T, H * Dv + 24, generator=g).to(dtype).cuda()
    lam, scale, eps = 0.7, 0.6, 1e-4
    aa = a.double().view(T, H, 2, Dp)[..., :Dv]
    o = aa[:, :, 0] - lam * aa[:, :, 1]
    want = o / torch.sqrt(o.pow(2).mean(-1, keepdim=True) + eps) * scale
    tol = dict(atol=2e-5, rtol=2e-5) if dtype == torch.float32 else dict(atol=1e-2, rtol=1e-2)
    out = torch.empty((T, H * Dv), dtype=dtype, device="cuda")
    for col in (8, 5):                                  # (logits from an aligned column and from any other)
        ops.differential_heads(a, rows, col, out, lam, scale, eps, H, Dv)
        gate = torch.sigmoid(rows.double()[:, col: col + H * Dv]).view(T, H, Dv)
        assert torch.allclose(out.double().view(T, H, Dv), want * gate, **tol)
    ops.differential_heads(a, None, 0, out, lam, scale, eps, H, Dv)
    assert torch.allclose(out.double().view(T, H, Dv), want, **tol)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T,E,ident,top,d,F", [(5, 4, 2, 2, 64, 32), (40, 6, 1, 1, 64, 40), (40, 5, 3, 3, 50, 9),
                                               (700, 8, 4, 2, 64, 64), (16, 3, 0, 3, 96, 24), (300, 70, 20, 4, 32, 16),
                                               (16, 1, 1, 2, 32, 8), (900, 6, 2, 4, 128, 64), (9, 10, 2, 9, 64, 16)])
def test_experts_with_corrected_choice_and_identity_experts(dtype, T, E, ident, top, d, F):
    """Every path of the experts' kernels (routing inside the grouping kernel for few tokens, tiles of 16, 64 and 128 rows
    on the matrix cores, the vector kernels) with choices by corrected shares and outputs that are the token itself."""
    from serve_amd import ops
    n = E + ident
    g = torch.Generator().manual_seed(T + E)
    h = torch.randn(T, d, generator=g).to(dtype)
    rw = (0.2 * torch.randn(n, d, generator=g)).to(dtype)
    corr = 0.3 * torch.randn(n, generator=g)
    W = {"router": rw.double(), "correction": corr.double()}
    wg, wu = ((torch.randn(E, F, d, generator=g) / d ** 0.5).to(dtype) for _ in range(2))
    wd = (torch.randn(E, d, F, generator=g) / F ** 0.5).to(dtype)
    for e in range(E):
        W.update({f"e{e}.gate": wg[e].double(), f"e{e}.up": wu[e].double(), f"e{e}.down": wd[e].double()})
    logits = (h.double() @ rw.double().T).float()
    ids_w, w_w = bp.route(h.double(), W, "", top)
    want = bp.experts_ff(h.double(), W, "", {"router": {"experts": E, "top": top}})
    choice = torch.sort(torch.softmax(logits.double(), -1) + corr.double(), dim=-1, descending=True).values
    clear = torch.ones(T, dtype=torch.bool) if top == n else (choice[:, top - 1] - choice[:, top]) > 1e-5
    clear &= (choice[:, :top].diff(dim=-1).abs() > 1e-6).all(-1) if top > 1 else True
    assert clear.float().mean().item() > 0.9
    ids = torch.empty((T, top), dtype=torch.int32, device="cuda")
    wts = torch.empty((T, top), dtype=torch.float32, device="cuda")
    yk = torch.full((T * top, d), float("nan"), dtype=torch.float32, device="cuda")
    gate_up = torch.stack([wg, wu]).cuda().contiguous()
    hc, wdc, lc, cc = h.cuda(), wd.cuda().contiguous(), logits.cuda().contiguous(), corr.cuda()
    if T <= ops.MOE_ROUTE_INSIDE:
        ops.moe_experts(hc, ids, gate_up[0], gate_up[1], wdc, yk, lc, wts, "all", 1.0, correction=cc, outputs=n)
    else:
        ops.moe_route(lc, n, top, ids, wts, "all", 1.0, cc)
        ops.moe_experts(hc, ids, gate_up[0], gate_up[1], wdc, yk, weights=wts, outputs=n)
    assert torch.equal(ids.cpu()[clear].long(), ids_w[clear])
    assert torch.allclose(wts.cpu()[clear].double(), w_w[clear], atol=1e-6)
    y = torch.empty((T, d), dtype=torch.float32, device="cuda")
    ops.moe_combine(yk, wts, None, None, n, y, ids, E, hc)
    err = (y.cpu().double() - want)[clear].norm(dim=-1) / want[clear].norm(dim=-1).clamp_min(1e-9)
    assert err.max().item() < (2e-5 if dtype == torch.float32 else 2e-2), err.max().item()


@pytest.mark.parametrize("d,dtype", [(64, torch.bfloat16), (50, torch.bfloat16), (64, torch.float32)])
def test_embedding_in_copies(d, dtype):
    from serve_amd import ops
    g = torch.Generator().manual_seed(d)
    E = torch.randn(37, d, generator=g).to(dtype).cuda()
    tok = torch.tensor([3, 36, 0, 5], dtype=torch.int32, device="cuda")
    x = torch.empty((4, 3, d), dtype=torch.float32, device="cuda")
    ops.embed(E, tok, x, scale=2.0)
    assert torch.equal(x, (2.0 * E[tok.long()].float())[:, None].expand(4, 3, d))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T,H,K,N", [(1, 3, 40, 24), (7, 2, 96, 64), (64, 4, 24, 16), (65, 4, 24, 16), (300, 2, 130, 70)])
def test_head_products_with_a_gate_per_head(dtype, T, H, K, N):
    """Both kernels (few tokens and many), with the gate's logits in any column of a wider product, and the latent cache
    write from a view of such a product."""
    from serve_amd import ops
    g = torch.Generator().manual_seed(T + K)
    x = torch.randn(T, H * (K + 5), generator=g).to(dtype).cuda()
    w = (torch.randn(H, K, N, generator=g) / K ** 0.5).to(dtype).cuda()
    rows = torch.randn(T, 3 + H + 2, generator=g).to(dtype).cuda()
    out = torch.empty((T, H * N), dtype=dtype, device="cuda")
    ops.head_linear(x, H * (K + 5), K + 5, w, out, H * N, N, T, gate_rows=rows, gate_col=3)
    xx = x.double().view(T, H, K + 5)[..., :K]
    want = torch.stack([xx[:, h] @ w[h].double() for h in range(H)], dim=1) * torch.sigmoid(rows.double()[:, 3: 3 + H])[..., None]
    tol = dict(atol=2e-5, rtol=2e-5) if dtype == torch.float32 else dict(atol=1e-2, rtol=1e-2)
    assert torch.allclose(out.double().view(T, H, N), want, **tol)
    R, dr, page, Dp = 20, 8, 4, 32
    wide = torch.randn(T, R + dr + 11, generator=g).to(dtype).cuda()
    nw = (1 + 0.1 * torch.randn(R, generator=g)).cuda()
    pos = torch.arange(T, dtype=torch.int32, device="cuda")
    P = -(-T // page)
    pages = []
    for z in (wide[:, 7: 7 + R + dr], wide[:, 7: 7 + R + dr].contiguous()):
        k, v = torch.zeros((P, 1, page, Dp), dtype=dtype, device="cuda"), torch.zeros((P, 1, Dp, page), dtype=dtype, device="cuda")
        ops.latent_kv_write(z, nw, pos, torch.ones(dr // 2, device="cuda"), pos, k, v, 1e-5, R, dr)
        pages.append((k, v))
    assert torch.equal(pages[0][0], pages[1][0]) and torch.equal(pages[0][1], pages[1][1]) and pages[0][0].abs().max() > 0
