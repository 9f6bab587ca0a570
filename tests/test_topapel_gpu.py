"""The Topapel decoder through the engine against the plain implementation, float32 and bfloat16: whole prompts and
first tokens; prompt then token by token; portions down to two tokens; unequal requests in one batch against each
alone, with pages and slots that are freed and used again; chunks' edges with sharp scores, in prompts and in
decoding; a far key among hundreds, at page borders; states over hundreds of tokens; long decoding; greedy generation
through the scheduler; the trace runner as a program; and the kernels alone."""
from __future__ import annotations

import os
import random
from types import SimpleNamespace

import pytest
import torch

from tests import topapel_models as tm
from tests.plain import topapel_plain as tp

pytestmark = pytest.mark.gpu

DTYPES = ["float32", "bfloat16"]
NAMES = ["TA", "TB", "TC", "TD", "TE", "TF"]
F64 = torch.float64


def tokens_for(n, seed, vocab):
    rng = random.Random(seed)
    return [rng.randrange(vocab) for _ in range(n)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_whole_prompts_and_first_tokens(tmp_path, name, dtype):
    folder = tm.make_folder(tmp_path, name)
    engine = tm.engine_for(folder, dtype)
    vocab = tm.MODELS[name][0].vocab
    for n in (1, 2, 3, 5, 61, 131):
        tokens = tokens_for(n, 100 + n, vocab)
        got = tm.run_portions(engine, f"r{n}", tokens, [n])
        tm.assert_rows_close(got, tm.plain_logits(folder, tokens), dtype, f"{name} whole {n}")
    engine.runner.cache.check_invariants()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_prompt_then_token_by_token(tmp_path, name, dtype):
    folder = tm.make_folder(tmp_path, name)
    engine = tm.engine_for(folder, dtype)
    vocab = tm.MODELS[name][0].vocab
    tokens = tokens_for(84, 7, vocab)
    want = tm.plain_logits(folder, tokens)
    got = tm.run_portions(engine, "r", tokens, [84 - 45] + [1] * 45)
    tm.assert_rows_close(got, want, dtype, f"{name} prompt + 45 single tokens")
    got = tm.run_portions(engine, "s", tokens[:30], [1] * 30)             # from the very first token on
    tm.assert_rows_close(got, want[:30], dtype, f"{name} token by token from the start")
    if dtype == "float32":
        whole = tm.run_portions(engine, "w", tokens, [84])
        assert tm.row_distance(got, whole[:30]).max().item() <= 3e-5


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_portions_of_changing_size(tmp_path, name, dtype):
    folder = tm.make_folder(tmp_path, name)
    engine = tm.engine_for(folder, dtype)
    vocab = tm.MODELS[name][0].vocab
    tokens = tokens_for(173, 8, vocab)
    want = tm.plain_logits(folder, tokens)
    for portions in ([7, 2, 16, 3, 2, 9, 2, 11, 5, 4, 1, 1, 2, 8, 100], [2] * 10 + [53, 17, 83], [1, 3, 169], [40, 33, 32, 68]):
        got = tm.run_portions(engine, "r", tokens, portions)
        tm.assert_rows_close(got, want, dtype, f"{name} portions {portions}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("page_size", [4, 16])
def test_chunks_edges_with_sharp_scores(tmp_path, dtype, page_size):
    """Outputs drawn wide, so that a key just inside or just outside a chunk (10 and 5 positions; a page holds 4 or 16)
    carries weight: the plain model moves by more than the bfloat16 tolerance when a chunk is one longer or shorter
    (see test_topapel_config.py).  Portions that end before, at and behind the chunks' edges, and single tokens across
    many of them; pages that no later token sees go back to the pool on the way."""
    folder = tm.make_folder(tmp_path, "TAsharp", config=tm.TA, seed=3, scales=tm.SHARP)
    engine = tm.engine_for(folder, dtype, num_pages=192 // page_size, page_size=page_size, debug_poison_cache=True)
    tokens = tokens_for(90, 21, tm.TA.vocab)
    want = tm.plain_logits(folder, tokens)
    for portions in ([90], [4, 1, 5, 1, 9, 10, 11, 2, 3] + [1] * 44, [9, 2] + [1] * 30 + [49], [5] * 18, [10] * 9):
        got = tm.run_portions(engine, "r", tokens, portions)
        tm.assert_rows_close(got, want, dtype, f"sharp chunks, portions {portions[:9]}...")
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
    folder = tm.make_folder(tmp_path, name)
    lengths = [23, 71, 9, 30, 117, 2, 36, 1, 60, 28, 33, 5]
    # four live requests: pool and slots are far fewer than the requests need together
    engine = tm.engine_for(folder, dtype, num_pages=71, page_size=4, max_requests=4, debug_poison_cache=True)
    vocab = tm.MODELS[name][0].vocab
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
            for page in (engine.runner.cache.block_table(k, 0) if engine.runner.cache.num_groups else []):
                pages_seen.setdefault(page, set()).add(k)
        for k in ended:
            engine.runner.release(k)
        engine.runner.cache.check_invariants()
    assert any(len(v) > 1 for v in slots_seen.values()), "no slot was used twice"
    assert name == "TE" or any(len(v) > 1 for p, v in pages_seen.items() if p >= 0), "no page went from one request to another"
    for k, toks in reqs.items():
        tm.assert_rows_close(torch.cat(rows[k]), tm.plain_logits(folder, toks), dtype, f"{name} request {k} in the mix")


def far_key_model(tmp_path, n, far, chunk):
    """One attention layer and an embedding table made so that one score stands out: the row of token 1 is set so that,
    behind the layer's norm, its query matrix (the queries' bias is zero here), the queries' norm and the rotation to
    position n - 1, the queries of both heads point along the rotated key of token 0 at position `far`.  A sequence
    that ends in token 1 and holds token 0 once, at `far`, then reads that key with nearly all of its weight."""
    from safetensors.torch import save_file
    cfg = tm.TopapelConfig(vocab=90, width=64, eps=1e-5, embedding_scale=1.0, logit_scale=0.8, logit_softcap=9.0, layers=(
        tm.L(tm.ATT(2, 1, 16, 1.2, chunk, tm.ROT(1000.0, 8, 3.0)), None),))
    folder = tm.make_folder(tmp_path, f"far{far}-{chunk}", config=cfg, seed=11, scales={r"q\.b$": 0.0, r"mix\.o$": 6.0})
    W = {k: v.double() for k, v in tm.plain_weights(folder).items()}
    f = tp.rotary_frequencies(8, 1000.0, {"factor": 3.0})
    h0 = tp.stream_norm(W["embed"][0:1], W["l0.norm1"], 1e-5)
    k0 = tp.over_rms((h0 @ W["l0.mix.k"].T + W["l0.mix.k.b"]).view(1, 1, 16), 1e-5) * W["l0.mix.k.norm"]
    k_at = tp.rotate(k0, torch.tensor([far]), f)
    q_plain = tp.rotate(k_at, torch.tensor([-(n - 1)]), f)[0, 0] / W["l0.mix.q.norm"]      # turning it to n - 1 gives k_at's direction
    h1 = torch.linalg.pinv(W["l0.mix.q"]) @ torch.cat([q_plain, q_plain])
    row = h1 / (1.0 + W["l0.norm1"])
    out = tm.plain_weights(folder)
    out["embed"][1] = (0.8 * row / row.pow(2).mean().sqrt()).to(out["embed"].dtype)     # (as large as the other rows)
    save_file({k: v.contiguous() for k, v in out.items()}, os.path.join(folder, "model.safetensors"))
    return folder


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_far_key_among_hundreds(tmp_path, dtype):
    rng = random.Random(5)
    n = 420
    # in the first page, further on, the last key of a page (page size 4); the first key of a chunk; the last of the
    # chunk before, which must not be seen
    for far, chunk in ((3, None), (37, None), (203, None), (210, 210), (209, 210), (400, 100), (399, 100)):
        folder = far_key_model(tmp_path, n, far, chunk)
        with_key = [rng.randrange(2, 90) for _ in range(n - 1)] + [1]
        with_key[far] = 0
        want = tm.plain_logits(folder, with_key)[-1:]
        seen = chunk is None or far // chunk == (n - 1) // chunk
        saved = tp.seen_keys
        try:                    # losing that one key, or seeing it, moves the last row by far more than the tolerance
            def other(T, c):
                s = saved(T, c).clone()
                s[-1, far] = not seen
                return s
            tp.seen_keys = other
            assert tm.row_distance(tm.plain_logits(folder, with_key)[-1:], want).item() > 2 * tm.TOLERANCE["bfloat16"]
        finally:
            tp.seen_keys = saved
        engine = tm.engine_for(folder, dtype, num_pages=120, page_size=4)
        got = tm.run_portions(engine, "r", with_key, [n - 3, 1, 1, 1])[-1:]
        tm.assert_rows_close(got, want, dtype, f"key {far} of {n}, chunks {chunk}, read by a token decoded alone")
        got = tm.run_portions(engine, "r", with_key, [200, 220])[-1:]
        tm.assert_rows_close(got, want, dtype, f"key {far} of {n}, chunks {chunk}, read from a portion")


@pytest.mark.parametrize("dtype", DTYPES)
def test_states_over_hundreds_of_tokens(tmp_path, dtype):
    """A linear attention that forgets nothing and a gated average that hardly moves (its gates' bias far below zero):
    the last of 400 tokens still rests on the first ones, whatever portions they came in."""
    cfg = tm.TopapelConfig(vocab=80, width=64, eps=1e-5, embedding_scale=1.0, logit_scale=0.7, logit_softcap=9.0, layers=(
        tm.L(tm.LIN(2, 32, 32, (1.0, 0.9995)), None), tm.L(tm.GRU(96), None)))
    folder = tm.make_folder(tmp_path, "states", config=cfg, seed=19, scales={r"mix\.o$": 4.0})
    from safetensors.torch import save_file
    W = tm.plain_weights(folder)
    W["l1.mix.z.b"] = (W["l1.mix.z.b"] - 6.0).contiguous()
    save_file(W, os.path.join(folder, "model.safetensors"))
    tokens = tokens_for(400, 41, 80)
    want = tm.plain_logits(folder, tokens)
    outer = tp.decayed_outer_products
    try:                            # (what losing the first 40 tokens of the state would do to the last rows)
        tp.decayed_outer_products = lambda q, k, v, a: torch.cat([outer(q[:40], k[:40], v[:40], a), outer(q[40:], k[40:], v[40:], a)])
        assert tm.row_distance(tm.plain_logits(folder, tokens)[-50:], want[-50:]).min().item() > 50 * tm.TOLERANCE["float32"]
    finally:
        tp.decayed_outer_products = outer
    engine = tm.engine_for(folder, dtype)
    for portions in ([400], [250] + [1] * 30 + [120], [3, 200, 5, 192], [17] * 23 + [9]):
        got = tm.run_portions(engine, "r", tokens, portions)
        tm.assert_rows_close(got, want, dtype, f"states, portions {portions[:4]}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["TA", "TB", "TC"])
def test_long_decoding(tmp_path, name, dtype):
    folder = tm.make_folder(tmp_path, name)
    engine = tm.engine_for(folder, dtype, num_pages=80)
    vocab = tm.MODELS[name][0].vocab
    tokens = tokens_for(260, 31, vocab)
    got = tm.run_portions(engine, "r", tokens, [4] + [1] * 256)
    tm.assert_rows_close(got, tm.plain_logits(folder, tokens), dtype, f"{name} 256 single tokens")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["TA", "TC", "TE"])
def test_greedy_generation_through_the_scheduler(tmp_path, name, dtype):
    """`generate` (scheduler, mixed steps, graphs, steps launched ahead of the host) picks the tokens the plain model
    picks, as long as the plain model's choice is clear."""
    from serve_amd.engine.engine import Request
    folder = tm.make_folder(tmp_path, name)
    engine = tm.engine_for(folder, dtype, num_pages=128, page_size=8, max_requests=3)
    vocab = tm.MODELS[name][0].vocab
    prompts = [tokens_for(n, 50 + n, vocab) for n in (5, 19, 1, 33, 8)]
    new = 12
    reqs = [Request(torch.tensor(p), len(p), new) for p in prompts]
    out = engine.generate(reqs, temperature=0.0, return_logits="all")
    compared = 0
    for p, o in zip(prompts, out):
        assert o.error is None and len(o.generated_tokens) == new
        seq = list(p)
        for i, tok in enumerate(o.generated_tokens.tolist()):
            row = tm.plain_logits(folder, seq)[-1]
            top2 = row.topk(2).values
            if (top2[0] - top2[1]).item() < (1e-3 if dtype == "float32" else 0.15) * row.std().item():
                break                            # the plain model's own choice is a close call: stop comparing
            assert tok == int(row.argmax()), f"{name}: token {i} after a prompt of {len(p)}"
            if dtype == "float32":
                tm.assert_rows_close(o.logits[i: i + 1], row[None], dtype, f"{name} logits of generated token {i}")
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
def test_graphs_give_what_eager_steps_give(tmp_path, dtype):
    """Decode steps and steps with prompt portions, replayed several times from graphs of padded shapes with other work
    between, against an engine that runs them kernel by kernel."""
    from serve_amd.engine.engine import Request
    folder = tm.make_folder(tmp_path, "TA")
    prompts = [tokens_for(n, 70 + n, tm.TA.vocab) for n in (12, 140, 3, 61, 90, 7, 33, 129)]
    outs = []
    for kw in (dict(use_graphs=False), dict(use_graphs=True), dict(use_graphs=True, graph_mixed_steps=True)):
        engine = tm.engine_for(folder, dtype, num_pages=256, page_size=8, max_requests=4, **kw)
        for _ in range(2):
            done = engine.generate([Request(torch.tensor(p), len(p), 20) for p in prompts], temperature=0.0)
        outs.append([o.generated_tokens.tolist() for o in done])
        engine.runner.cache.check_invariants()
    if dtype == "float32":
        assert outs[0] == outs[1] == outs[2]
    else:
        # (padded shapes may sum a product's parts in another order: a close call may fall the other way, no more)
        for other in outs[1:]:
            same = sum(a == b for x, y in zip(outs[0], other) for a, b in zip(x, y))
            assert same >= 0.6 * 20 * len(prompts)


@pytest.mark.parametrize("dtype", DTYPES)
def test_traces_through_the_program(tmp_path, dtype):
    """`bin/trace_run` as a child process on a model folder: whole prompts, prompt then single tokens, portions, and a
    mix of four live requests (four state slots, pages for 256 tokens), against the plain model."""
    import json
    import subprocess
    import numpy as np
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    name = "TA"
    folder = tm.make_folder(tmp_path, name)
    vocab = tm.MODELS[name][0].vocab
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
        tm.assert_rows_close(torch.cat(rows[k]), tm.plain_logits(folder, t), dtype, f"trace request {k}")


def test_generate_from_the_command_line():
    """`python -m serve_amd generate` with the named shape: as many token lists as prompts, of the asked length."""
    import json
    import subprocess
    import sys
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    proc = subprocess.run([sys.executable, "-m", "serve_amd", "generate", "--shape", "topapel-tiny", "--random-prompts", "3:30",
                           "--max-new-tokens", "6", "--temperature", "0.7"], cwd=root, capture_output=True, text=True, timeout=600)
    assert proc.returncode == 0, proc.stderr[-3000:]
    lines = [json.loads(l) for l in proc.stdout.splitlines() if l.startswith("[")]
    assert len(lines) == 3 and all(len(l) == 6 and all(0 <= t < 512 for t in l) for l in lines)


# ---------------------------------------------------------------------------------------------
# the kernels alone
# ---------------------------------------------------------------------------------------------
def i32(v):
    return torch.tensor(v, dtype=torch.int32, device="cuda")


def step_of(lens, slots=None, ctx_lens=None):
    """What the kernels read of a step of segments with the given lengths."""
    cu = [0]
    for n in lens:
        cu.append(cu[-1] + n)
    ctx_lens = list(lens) if ctx_lens is None else list(ctx_lens)
    return SimpleNamespace(num_tokens=cu[-1], num_segments=len(lens), cu_q=i32(cu), ctx_len=i32(ctx_lens),
                           seg_of_token=i32([i for i, n in enumerate(lens) for _ in range(n)]),
                           state_slots=i32(list(range(len(lens))) if slots is None else slots), q_lens=list(lens),
                           ctx_lens=ctx_lens, max_q_len=max(lens), max_ctx_len=max(ctx_lens), decode_only=max(lens) == 1)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,D,page,chunk", [(4, 2, 32, 4, 10), (9, 3, 80, 16, 72), (3, 1, 16, 12, 33), (8, 1, 128, 32, 100), (2, 2, 136, 8, 40),
                                              (20, 1, 64, 16, 48), (2, 1, 64, 16, 1), (4, 4, 48, 16, 4096)])
def test_attention_in_chunks(dtype, H, G, D, page, chunk):
    """Every attention kernel (a wave a row; tiles and single tokens in float32; one wave, one workgroup and prompt
    tiles on the matrix cores, with keys cut into parts) under a mask of chunks, with sinks and with NaN in every place
    that no token of the step may see."""
    from serve_amd import ops
    g = torch.Generator().manual_seed(H * D + chunk)
    cases = [([1] * 5, [1, chunk, chunk + 1, 2 * chunk + 3, 700]), ([1, 1, 1, 1, 37, 2, 150], [300, 9, 65, 641, 37, 66, 400]),
             ([1] * 40, [7 * i + 1 for i in range(40)]), ([130], [1000]), ([9], [64])]
    for lens, ctxs in cases:
        ctxs = [max(c, n) for c, n in zip(ctxs, lens)]
        step = step_of(lens, None, ctxs)
        T, B, MP = step.num_tokens, len(lens), -(-max(ctxs) // page)
        order = torch.randperm(B * MP, generator=g).tolist()
        bt = torch.tensor(order, dtype=torch.int32).view(B, MP)
        k = torch.full((B * MP, G, page, D), float("nan"))
        v = torch.full((B * MP, G, D, page), float("nan"))
        q = torch.randn(T, H, D, generator=g).to(dtype)
        sinks = torch.randn(H, generator=g)
        scale, want, at = 2.0 / D ** 0.5, torch.zeros(T, H, D, dtype=F64), 0
        for b, (n, c) in enumerate(zip(lens, ctxs)):
            first = (c - n) // chunk * chunk                    # the first key that any token of the segment sees
            kk = torch.randn(c, G, D, generator=g).to(dtype)
            vv = torch.randn(c, G, D, generator=g).to(dtype)
            for p in range(first, c):
                k[bt[b, p // page], :, p % page] = kk[p].float()
                v[bt[b, p // page], :, :, p % page] = vv[p].float()
            seen = tp.seen_keys(c, chunk)[c - n:]
            for h in range(H):
                s = q[at: at + n, h].double() @ kk[:, h // (H // G)].double().T * scale
                want[at: at + n, h] = tp.sink_softmax(s, seen, sinks[h].double()) @ vv[:, h // (H // G)].double()
            at += n
        qc, kc, vc = q.reshape(T, H * D).cuda(), k.to(dtype).cuda(), v.to(dtype).cuda()
        out = torch.empty((T, H * D), dtype=dtype, device="cuda")
        tol = dict(atol=2e-5, rtol=2e-5) if dtype == torch.float32 else dict(atol=3e-2, rtol=2e-2)
        bt = bt.cuda()
        ops.paged_attention(qc, H * D, out, kc, vc, bt, step, H, scale, None, sinks.cuda(), chunk)
        got = out.view(T, H, D).double().cpu()
        assert torch.allclose(got, want, **tol), (lens, ctxs, (got - want).abs().max().item())
        ops.paged_attention_simple(qc, H * D, out, kc, vc, bt, step.cu_q, step.ctx_len, step.seg_of_token, T, H, scale, None,
                                   sinks.cuda(), chunk)
        assert torch.allclose(out.view(T, H, D).double().cpu(), want, **tol)
        # the key range cut into parts, some of which see nothing
        if dtype == torch.bfloat16 and ops.mfma_attention_available(qc, kc, H * D, scale):
            for splits in (2, 5):
                ops.paged_attention_mfma(qc, H * D, out, kc, vc, bt, step.cu_q, step.ctx_len, T, max(lens), H, scale, None,
                                         splits, sinks=sinks.cuda(), chunk=chunk)
                assert torch.allclose(out.view(T, H, D).double().cpu(), want, **tol)
        elif dtype == torch.float32 and ops.tiled_attention_available(qc, kc, H * D):
            for splits in (1, 3):
                ops.paged_attention_tiled_f32(qc, H * D, out, kc, vc, bt, step.cu_q, step.ctx_len, T, max(lens), H, scale,
                                              None, splits, sinks.cuda(), chunk)
                assert torch.allclose(out.view(T, H, D).double().cpu(), want, **tol)
                if max(lens) == 1:
                    ops.paged_attention_decode_f32(qc, H * D, out, kc, vc, bt, step.cu_q, step.ctx_len, H, scale, None,
                                                   splits, 0, sinks.cuda(), chunk)
                    assert torch.allclose(out.view(T, H, D).double().cpu(), want, **tol)
    with pytest.raises(ops.KernelError, match="not both"):
        ops.paged_attention(qc, H * D, out, kc, vc, bt, step, H, scale, 8, sinks.cuda(), chunk)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,D,Dp,rot,shared,T", [
    (4, 2, 32, 32, 16, True, 11), (9, 3, 80, 80, 80, True, 40), (3, 3, 10, 16, 4, True, 11), (2, 1, 136, 144, 64, True, 11),
    (5, 1, 24, 32, 24, True, 33), (4, 4, 16, 16, 0, True, 11), (3, 1, 64, 64, 32, False, 70), (2, 2, 20, 32, 6, False, 11),
    (8, 2, 128, 128, 128, True, 300), (2, 1, 8, 16, 2, True, 11)])
def test_norm_rotation_and_cache_write(dtype, H, G, D, Dp, rot, shared, T):
    """Both kernels (eight dims a lane from aligned rows; a wave a head at any size): biases, norm per head, rotation, and
    values that are the keys as projected or have columns of their own."""
    from serve_amd import ops
    page = 4
    P = (T + 30) // page + 2
    g = torch.Generator().manual_seed(H * D + rot + T)
    cols = H * D + G * D * (1 if shared else 2)
    z = torch.randn(T, cols + (8 if H % 2 == 0 else 5), generator=g).to(dtype).cuda()       # (rows wider than what is read)
    bias = torch.randn(cols, generator=g)
    wq, wk = 1 + 0.3 * torch.randn(D, generator=g), 1 + 0.3 * torch.randn(D, generator=g)
    pos = torch.tensor([(37 * t) % 900 for t in range(T)])
    slot_l = [-1 if t % 10 == 7 else t + 12 for t in range(T)]
    f = tp.rotary_frequencies(rot, 100.0, {"factor": 2.5}) if rot else torch.zeros(0, dtype=F64)
    inv = f.float().cuda() if rot else None
    eps = 1e-3
    for with_bias in (True, False):
        k_pages = torch.full((P, G, page, Dp), 9.0, dtype=dtype, device="cuda")
        v_pages = torch.full((P, G, Dp, page), 9.0, dtype=dtype, device="cuda")
        q = torch.full((T, H * Dp), 9.0, dtype=dtype, device="cuda")
        args = dict(bias=bias.cuda() if with_bias else None, inv_freq=inv, rot_dim=rot, values_are_keys=shared)
        ops.qk_norm_kv_write(z, q, i32(pos.tolist()), i32(slot_l), k_pages, v_pages, wq.cuda(), wk.cuda(), eps, H, G, D, D, **args)
        zz = z[:, :cols].double().cpu() + (bias.double() if with_bias else 0.0)
        raw_k = zz[:, H * D: (H + G) * D].reshape(T, G, D)
        qn = tp.over_rms(zz[:, : H * D].reshape(T, H, D), eps) * wq.double()
        kn = tp.over_rms(raw_k, eps) * wk.double()
        if rot:
            qn, kn = tp.rotate(qn, pos, f), tp.rotate(kn, pos, f)
        vn = raw_k if shared else zz[:, (H + G) * D:].reshape(T, G, D)
        tol = dict(atol=2e-4, rtol=2e-5) if dtype == torch.float32 else dict(atol=3e-2, rtol=2e-2)
        qq = q.view(T, H, Dp).double().cpu()
        assert torch.allclose(qq[..., :D], qn, **tol) and (qq[..., D:] == 0).all()
        stored = [t for t in range(T) if slot_l[t] >= 0]
        st = torch.tensor([slot_l[t] for t in stored])
        kk, vv = k_pages.double().cpu()[st // page, :, st % page], v_pages.double().cpu()[st // page, :, :, st % page]
        assert torch.allclose(kk[..., :D], kn[stored], **tol) and (kk[..., D:] == 0).all()
        assert torch.allclose(vv[..., :D], vn[stored], **tol) and (vv[..., D:] == 0).all()
        used = torch.zeros(P * page, dtype=torch.bool)
        used[st] = True
        free = (~used).nonzero()[:, 0]
        assert (k_pages.cpu()[free // page, :, free % page] == 9).all()
        assert (v_pages.cpu()[free // page, :, :, free % page] == 9).all()
        q2 = torch.empty_like(q)
        ops.qk_norm_kv_write(z, q2, i32(pos.tolist()), None, None, None, wq.cuda(), wk.cuda(), eps, H, G, D, D, **args)
        assert torch.equal(q2, q)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T,d,parts", [(3, 50, 2), (70, 64, 1), (5, 2304, 4), (2, 8200, 1), (300, 512, 8)])
def test_a_row_that_joins_the_stream_behind_the_norm(dtype, T, d, parts):
    from serve_amd import ops
    g = torch.Generator().manual_seed(d)
    x0 = torch.randn(T, d, generator=g)
    w, b = torch.randn(d, generator=g), torch.randn(d, generator=g)
    delta = torch.randn(parts, T, d, generator=g)
    for dl in (delta, None):
        x, out = x0.cuda(), torch.empty((T, d), dtype=dtype, device="cuda")
        ops.add_rmsnorm(x, None if dl is None else dl.cuda(), w.cuda(), 1e-5, out, after=b.cuda())
        v = x0.double() + (dl.double().sum(0) if dl is not None else 0.0)
        assert torch.allclose(x.double().cpu(), v + b.double(), atol=1e-5, rtol=1e-6)
        want = tp.over_rms(v, 1e-5) * w.double()
        assert torch.allclose(out.double().cpu(), want, **(dict(atol=2e-5, rtol=2e-5) if dtype == torch.float32 else dict(atol=2e-2, rtol=1e-2)))
    with pytest.raises(ops.KernelError):
        ops.add_rmsnorm(x, None, w.cuda(), 1e-5, torch.empty((1, d), dtype=dtype, device="cuda"), i32([0]), b.cuda())


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T,n,parts", [(1, 4, 1), (3, 27, 1), (5, 27, 3), (9, 96, 2), (300, 8192, 1), (7, 14336, 4), (2, 33000, 1), (40, 2100, 8),
                                       (600, 1001, 1)])
def test_polynomial_of_normed_powers(dtype, T, n, parts):
    from serve_amd import ops
    g = torch.Generator().manual_seed(n + T)
    z = 2.0 * torch.randn(parts, T, n, generator=g)
    coef = torch.tensor([0.5, -0.7, 0.9, 0.3])
    tol = dict(atol=3e-5, rtol=3e-5) if dtype == torch.float32 else dict(atol=1e-2, rtol=1e-2)
    out = torch.empty((T, n), dtype=dtype, device="cuda")
    ops.poly_norm(z.cuda(), coef.cuda(), 0.01, out)
    assert torch.allclose(out.double().cpu(), tp.poly_norm(z.double().sum(0), coef.double(), 0.01), **tol)
    one = z[0].to(dtype)
    ops.poly_norm(one.cuda(), coef.cuda(), 1e-6, out)
    assert torch.allclose(out.double().cpu(), tp.poly_norm(one.double(), coef.double(), 1e-6), **tol)


def test_scaled_and_capped_logits():
    from serve_amd import ops
    g = torch.Generator().manual_seed(4)
    for R, V in ((1, 5), (3, 513), (2, 40000)):
        y = 30.0 * torch.randn(R, V, generator=g)
        got = ops.scale_soft_cap(y.cuda(), 0.4, 12.0).double().cpu()
        assert torch.allclose(got, tp.soft_cap(0.4 * y.double(), 12.0), atol=1e-5, rtol=1e-5)
        assert torch.allclose(ops.scale_soft_cap(y.cuda(), 0.25, 0.0).cpu(), 0.25 * y)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,dk,dv", [(2, 16, 72), (3, 24, 40), (4, 128, 128), (2, 136, 24), (1, 1, 1), (6, 48, 32)])
@pytest.mark.parametrize("lens", [[1, 1, 1], [3, 1, 5], [40, 1, 2, 17], [700], [16, 300, 1, 1]])
def test_recurrence_with_one_decay_a_head(dtype, H, dk, dv, lens):
    """Constant decays and z sigmoid(z) on q, k and v, over two steps of the same requests (short and long segments, long
    ones cut into pieces; a segment of no request keeps nothing)."""
    from serve_amd import ops
    g = torch.Generator().manual_seed(H * dk + dv + sum(lens))
    decay = torch.tensor([1.0, 1e-6, 0.5, 0.97, 0.999, 1e-30][:H], dtype=F64)
    B, T = len(lens), sum(lens)
    slots = [2 * b for b in range(B)]
    if B > 2:
        slots[1] = -1
    state = torch.zeros(2 * B, ops.decay_scan_state_floats(H, dk, dv), device="cuda")
    past = [[] for _ in range(B)]
    step = step_of(lens, slots)
    silu = lambda t: t * torch.sigmoid(t)                                                  # noqa: E731
    for turn in range(2):
        z = torch.randn(T, H * (2 * dk + dv) + 3, generator=g).to(dtype)
        zc = z.cuda()
        out = torch.empty((T, H * dv), dtype=torch.float32, device="cuda")
        ops.decay_scan(zc[:, : H * dk], zc[:, H * dk: 2 * H * dk], zc[:, 2 * H * dk: H * (2 * dk + dv)], decay.log().float().cuda(),
                       state, 0, step, out, H, H, dk, dv, silu=True)
        at = 0
        for b, n in enumerate(lens):
            rows = z[at: at + n].double()
            past[b] = [rows] if slots[b] < 0 else past[b] + [rows]
            r = silu(torch.cat(past[b]))
            m = r.shape[0]
            want = tp.decayed_outer_products(r[:, : H * dk].reshape(m, H, dk), r[:, H * dk: 2 * H * dk].reshape(m, H, dk),
                                             r[:, 2 * H * dk: H * (2 * dk + dv)].reshape(m, H, dv), decay)[-n:].reshape(n, H * dv)
            got = out[at: at + n].double().cpu()
            # (per token and head: sums over hundreds of tokens of values of order one)
            scale = want.view(n, H, dv).pow(2).mean(-1, keepdim=True).sqrt().clamp_min(0.1)
            assert ((got - want).view(n, H, dv) / scale).abs().max().item() < 3e-4, (turn, b)
            at += n
    assert (state[1::2] == 0).all()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("n", [120, 2048, 2500])
def test_read_out_norm_with_a_sigmoid_gate(dtype, n):
    from serve_amd import ops
    g = torch.Generator().manual_seed(n)
    T = 7
    o = 3.0 * torch.randn(T, n, generator=g)
    rows = torch.randn(T, n + 11, generator=g).to(dtype)
    w = 1 + 0.2 * torch.randn(n, generator=g)
    y = torch.empty((T, n), dtype=dtype, device="cuda")
    ops.gated_group_norm(o.cuda(), rows.cuda(), 11, w.cuda(), n, False, 1e-4, y, gate="sigmoid")
    want = tp.over_rms(o.double(), 1e-4) * w.double() * torch.sigmoid(rows[:, 11:].double())
    assert torch.allclose(y.double().cpu(), want, **(dict(atol=1e-5, rtol=1e-5) if dtype == torch.float32 else dict(atol=2e-2, rtol=1e-2)))
    with pytest.raises(ops.KernelError, match="gate"):
        ops.gated_group_norm(o.cuda(), rows.cuda(), 11, w.cuda(), n, False, 1e-4, y, gate="other")


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("W", [1, 37, 300, 2048])
@pytest.mark.parametrize("parts", [1, 3, 8])
@pytest.mark.parametrize("lens", [[1, 1, 1], [3, 1, 16], [31, 1, 33], [32, 32, 64], [5, 1, 200, 1, 1, 40], [500], [1] * 50 + [17, 90]])
def test_gated_average_over_steps(dtype, W, parts, lens):
    """Segment by segment and over tiles of 32 tokens that lie across the segments' borders, over two steps of the same
    requests; partial sums; a segment of no request keeps nothing; places behind the state's row are left alone."""
    from serve_amd import ops
    g = torch.Generator().manual_seed(W + parts + sum(lens))
    B, T = len(lens), sum(lens)
    slots = [2 * b for b in range(B)]
    if B > 2:
        slots[1] = -1
    state = torch.zeros(2 * B, W + 3, device="cuda")
    bias = torch.randn(2 * W, generator=g)
    past = [[] for _ in range(B)]
    step = step_of(lens, slots)
    for turn in range(2):
        rows = torch.randn(parts, T, 3 * W, generator=g)
        rows[..., :W] -= 1.0 / parts                        # (gates below one half: states that last)
        y = torch.empty((T, W), dtype=dtype, device="cuda")
        ops.gated_average(rows.cuda() if parts > 1 else rows[0].contiguous().cuda(), bias.cuda(), state, step, y)
        total, at = rows.double().sum(0), 0
        for b, n in enumerate(lens):
            r = total[at: at + n]
            past[b] = [r] if slots[b] < 0 else past[b] + [r]
            r = torch.cat(past[b])
            S = tp.gated_average(torch.sigmoid(r[:, :W] + bias[:W].double()), tp.positive_part(r[:, W: 2 * W] + bias[W:].double()))
            want = (S * tp.silu(r[:, 2 * W:]))[-n:]
            tol = dict(atol=2e-5, rtol=2e-5) if dtype == torch.float32 else dict(atol=1e-2, rtol=1e-2)
            assert torch.allclose(y[at: at + n].double().cpu(), want, **tol), (turn, b)
            if slots[b] >= 0:
                assert torch.allclose(state[slots[b], :W].double().cpu(), S[-1], atol=1e-5, rtol=1e-5)
            at += n
    assert (state[1::2] == 0).all() and (state[:, W:] == 0).all()
