"""Offline batch benchmark in the manner of the reference's only command-line program,
`python3 serve/benchmark.py [--profile] [--profile-only]` (serve/benchmark.py:27-103): seeded
random requests (input and output lengths uniform in 1..N, token ids below 10000,
serve/benchmark.py:12-24), one warm-up run of `generate`, one timed run, tokens per second, and
an optional profiler trace.

What the reference fixes by editing its source is an option here: the model (a folder, or a
named shape with random weights), dtype, lengths, number of sequences, temperature.

    python -m serve_amd.benchmark --shape llama-1b --num-sequences 256
    python -m serve_amd.benchmark --model /path/to/folder --dtype float32 --profile
"""
from __future__ import annotations

import argparse
import random
import sys
import time

import torch

from .config.engine import EngineConfig
from .config.llama import Llama3RopeScaling, LlamaConfig

_L3 = lambda factor: Llama3RopeScaling(factor, 1.0, 4.0, 8192)   # noqa: E731

# named shapes with random weights (the two the reference knows, serve/utils.py:11-38, and two more)
SHAPES = {
    "tiny": LlamaConfig(vocab_size=10000, hidden_size=64, intermediate_size=192, num_hidden_layers=2,
                        num_attention_heads=4, num_key_value_heads=2, head_dim=16),
    # the two tiny configurations that the engine's equality checks are specified on
    "tiny-a": LlamaConfig(vocab_size=256, hidden_size=64, intermediate_size=192, num_hidden_layers=2,
                          num_attention_heads=4, num_key_value_heads=2, head_dim=16, rms_norm_eps=1e-5,
                          rope_theta=10000.0, tie_word_embeddings=False),
    "tiny-b": LlamaConfig(vocab_size=512, hidden_size=96, intermediate_size=256, num_hidden_layers=3,
                          num_attention_heads=3, num_key_value_heads=1, head_dim=32, rms_norm_eps=1e-6,
                          rope_theta=500000.0, rope_scaling=Llama3RopeScaling(32.0, 1.0, 4.0, 64),
                          tie_word_embeddings=True),
    "llama-1b": LlamaConfig(vocab_size=128256, hidden_size=2048, intermediate_size=8192, num_hidden_layers=16,
                            num_attention_heads=32, num_key_value_heads=8, head_dim=64, rope_theta=500000.0,
                            rope_scaling=_L3(32.0), tie_word_embeddings=True),
    "llama-3b": LlamaConfig(vocab_size=128256, hidden_size=3072, intermediate_size=8192, num_hidden_layers=28,
                            num_attention_heads=24, num_key_value_heads=8, head_dim=128, rope_theta=500000.0,
                            rope_scaling=_L3(32.0), tie_word_embeddings=True),
    "llama-8b": LlamaConfig(vocab_size=128256, hidden_size=4096, intermediate_size=14336, num_hidden_layers=32,
                            num_attention_heads=32, num_key_value_heads=8, head_dim=128, rope_theta=500000.0,
                            rope_scaling=_L3(8.0), tie_word_embeddings=False),
}


def _zozosun_shape(width: int, vocab: int, groups: int, delta_heads: int, attn_heads: int, ff: int, experts: int,
                   top: int, expert_ff: int, shared_ff: int, window: int):
    """A Zozosun shape at the sizes of a real model's layers: `groups` times four layers, delta rule + dense,
    delta rule + experts, latent attention + dense, latent attention on the cache of the layer before + experts.
    The latent row (kv_rank 96 + 32 rotated dims) is as wide as the matrix-core attention's widest head."""
    from .config.zozosun import (DeltaMixerConfig, DenseMlpConfig, LatentMixerConfig, MoeMlpConfig, ZozosunConfig,
                                 ZozosunLayerConfig)
    delta = DeltaMixerConfig(heads=delta_heads, kv_heads=delta_heads // 2, dim=128, vdim=128, conv=4)
    layers = []
    for g in range(groups):
        latent = LatentMixerConfig(heads=attn_heads, dim=64, rot_dim=32, vdim=64, kv_rank=96, scale=96 ** -0.5,
                                   rot_base=1.0e6, window=window)
        reader = LatentMixerConfig(heads=attn_heads, dim=64, rot_dim=32, vdim=64, kv_rank=96, scale=96 ** -0.5,
                                   rot_base=1.0e6, window=window, kv_from=4 * g + 2)
        moe = MoeMlpConfig(experts, top, expert_ff, shared_ff)
        layers += [ZozosunLayerConfig(delta, DenseMlpConfig(ff)), ZozosunLayerConfig(delta, moe),
                   ZozosunLayerConfig(latent, DenseMlpConfig(ff)), ZozosunLayerConfig(reader, moe)]
    return ZozosunConfig(vocab=vocab, width=width, eps=1e-5, layers=tuple(layers))


# Zozosun at two widths, and beside each a Llama shape of the same width, depth, vocabulary and feed-forward
# width (the closest model the engine has): `bench.py --designs` measures them side by side
SHAPES.update({
    "zozosun-tiny": _zozosun_shape(64, 512, 1, 2, 2, 128, 4, 2, 32, 64, 24),
    "zozosun-2k": _zozosun_shape(2048, 32768, 2, 16, 16, 8192, 32, 4, 1024, 2048, 1024),
    "zozosun-4k": _zozosun_shape(4096, 32768, 1, 32, 32, 14336, 64, 6, 1536, 3072, 1024),
    "llama-2k": LlamaConfig(vocab_size=32768, hidden_size=2048, intermediate_size=8192, num_hidden_layers=8,
                            num_attention_heads=32, num_key_value_heads=8, head_dim=64, rope_theta=500000.0),
    "llama-4k": LlamaConfig(vocab_size=32768, hidden_size=4096, intermediate_size=14336, num_hidden_layers=4,
                            num_attention_heads=32, num_key_value_heads=8, head_dim=128, rope_theta=500000.0),
})


def _timopel_shape(width: int, vocab: int, layers: int, heads: int, kv_heads: int, head: int, ff: int, experts: int,
                   top: int, expert_ff: int, shared_ff: int):
    """A Timopel shape at the sizes of a real model's layers: attention layers with `heads` on `kv_heads` heads of
    `head` (keys and values alike), whose feed-forwards are in turn dense and routed experts with a shared one; all
    layers but the first blend their values with the first layer's."""
    from .config.timopel import (ClampedMoeConfig, GatedDenseConfig, QueryTemperature, SinkAttentionConfig,
                                 TimopelConfig, TimopelLayerConfig)
    mixer = SinkAttentionConfig(heads, kv_heads, head, head, head ** -0.5, QueryTemperature(0.1, 1024), True)
    moe = ClampedMoeConfig(experts, top, 1.0, expert_ff, 7.0, shared_ff, 7.0)
    return TimopelConfig(vocab=vocab, width=width, eps=1e-5, residual_mult=0.5, embedding_scale=1.0,
                         layers=tuple(TimopelLayerConfig(mixer, GatedDenseConfig(ff) if i % 2 == 0 else moe)
                                      for i in range(layers)))


# Timopel at the same two widths, depths, vocabularies, head shapes and dense feed-forward widths as the Llama
# shapes above (its experts as Zozosun's)
SHAPES.update({
    "timopel-tiny": _timopel_shape(64, 512, 2, 4, 2, 16, 128, 4, 2, 32, 64),
    "timopel-2k": _timopel_shape(2048, 32768, 8, 32, 8, 64, 8192, 32, 4, 1024, 2048),
    "timopel-4k": _timopel_shape(4096, 32768, 4, 32, 8, 128, 14336, 64, 6, 1536, 3072),
})


def _kotipel_shape(width: int, vocab: int, layers: int, loop, heads: int, kv_heads: int, head: int, lin_heads: int,
                   lin_dim: int, lin_vdim: int, ssm_heads: int, ssm_groups: int, ff: int, side: int):
    """A Kotipel shape at the sizes of a real model's layers: in turn a parallel layer (softmax attention with `heads` on
    `kv_heads` heads of `head`, half of whose dims are rotated, beside a gated linear attention of `lin_heads` heads of
    `lin_dim` x `lin_vdim`) and a state-space layer (inner width twice the model's: `ssm_heads` heads of 64, state 128,
    four taps), each with a clamped feed-forward of `ff` and a token input of `side`; `loop` = (start, stop, times)."""
    from .config.kotipel import (ClampedDenseConfig, GatedAttentionConfig, KotipelConfig, KotipelLayerConfig,
                                 LinearAttentionConfig, LoopConfig, ParallelMixerConfig, RotScaling, StateSpaceMixerConfig)
    par = ParallelMixerConfig(
        GatedAttentionConfig(heads, kv_heads, head, head, head ** -0.5, head // 2, 500000.0, RotScaling(8.0, 1.0, 4.0, 8192.0)),
        LinearAttentionConfig(lin_heads, lin_dim, lin_vdim, 16.0, 16))
    ssm = StateSpaceMixerConfig(ssm_heads, 64, 128, ssm_groups, 4, 1)
    mlp = ClampedDenseConfig(ff, 7.0)
    return KotipelConfig(vocab=vocab, width=width, eps=1e-5, loop=LoopConfig(*loop), side_dim=side,
                         layers=tuple(KotipelLayerConfig(par if i % 2 == 0 else ssm, mlp) for i in range(layers)))


# Kotipel at the same two widths, vocabularies, attention head shapes and feed-forward widths; with the layers that
# run twice it has as many layer runs as the Llama shapes have layers (8 and 4)
SHAPES.update({
    "kotipel-tiny": _kotipel_shape(64, 512, 2, (0, 2, 2), 4, 2, 16, 2, 16, 32, 2, 1, 128, 8),
    "kotipel-2k": _kotipel_shape(2048, 32768, 6, (2, 4, 2), 32, 8, 64, 16, 64, 128, 64, 1, 8192, 256),
    "kotipel-4k": _kotipel_shape(4096, 32768, 3, (1, 2, 2), 32, 8, 128, 16, 128, 256, 128, 8, 14336, 256),
})


def _robuvik_shape(width: int, vocab: int, layers: int, loop, heads: int, kv_heads: int, head: int, window: int,
                   q_rank: int, ff: int, experts: int, top: int, expert_ff: int, shared_ff: int, buckets: int):
    """A Robuvik shape at the sizes of a real model's layers: in turn an attention layer (`heads` on `kv_heads` heads
    of `head`, all dims rotated with stretched frequencies, a window, biases, a sink) with a dense feed-forward of
    `ff`, and a latent-attention layer (`heads` heads of 64 + 32 rotated dims over a latent of 96: a cache row as
    wide as the matrix-core attention's widest head; queries through a latent of `q_rank`) with routed experts and a
    shared one; `loop` = (start, stop, times); a pair table of `buckets` rows."""
    from .config.kotipel import LoopConfig
    from .config.robuvik import (BigramConfig, DenseConfig, ExpertsConfig, LatentAttentionConfig, RobuvikConfig,
                                 RobuvikLayerConfig, RotConfig, WindowAttentionConfig, YarnScaling)
    yarn = YarnScaling(4.0, 2048.0, 32.0, 1.0)
    att = WindowAttentionConfig(heads, kv_heads, head, head, head ** -0.5, RotConfig(500000.0, head, yarn), window)
    lat = LatentAttentionConfig(heads, 64, 32, 64, 96, q_rank, 96 ** -0.5, RotConfig(1.0e6, 32, yarn))
    moe = ExpertsConfig(experts, top, expert_ff, shared_ff)
    return RobuvikConfig(vocab=vocab, width=width, eps=1e-5, bigram=BigramConfig(buckets, 37, 11), loop=LoopConfig(*loop),
                         layers=tuple(RobuvikLayerConfig(att, DenseConfig(ff)) if i % 2 == 0 else RobuvikLayerConfig(lat, moe)
                                      for i in range(layers)))


# Robuvik at the same two widths, vocabularies, attention head shapes and dense feed-forward widths (its experts as
# Zozosun's and Timopel's); with the layers that run twice it has as many layer runs as the Llama shapes have layers
SHAPES.update({
    "robuvik-tiny": _robuvik_shape(64, 512, 2, (0, 2, 2), 4, 2, 16, 24, 32, 128, 4, 2, 32, 64, 251),
    "robuvik-2k": _robuvik_shape(2048, 32768, 6, (2, 4, 2), 32, 8, 64, 1024, 512, 8192, 32, 4, 1024, 2048, 65521),
    "robuvik-4k": _robuvik_shape(4096, 32768, 3, (1, 2, 2), 32, 8, 128, 1024, 1024, 14336, 64, 6, 1536, 3072, 65521),
})


def _topapel_shape(width: int, vocab: int, layers: int, heads: int, kv_heads: int, head: int, chunk: int, gru: int,
                   lin_heads: int, lin_dim: int, ff: int):
    """A Topapel shape at the sizes of a real model's layers: in turn an attention layer (`heads` on `kv_heads` heads of
    `head`, all dims rotated, chunks of `chunk`), a gated average of `gru` channels and a linear attention of `lin_heads`
    heads of `lin_dim` x `lin_dim` with decays from 0.9 to 0.999, each with a feed-forward of `ff`."""
    from .config.topapel import (ChunkAttentionConfig, LightningConfig, LinearRotConfig, MinGruConfig, TopapelConfig,
                                 TopapelLayerConfig)
    step = (0.999 - 0.9) / max(lin_heads - 1, 1)
    mixers = (ChunkAttentionConfig(heads, kv_heads, head, head ** -0.5, chunk, LinearRotConfig(500000.0, head, 4.0)),
              MinGruConfig(gru),
              LightningConfig(lin_heads, lin_dim, lin_dim, tuple(round(0.9 + step * h, 6) for h in range(lin_heads))))
    return TopapelConfig(vocab=vocab, width=width, eps=1e-5, embedding_scale=width ** 0.5, logit_scale=1.0, logit_softcap=30.0,
                         layers=tuple(TopapelLayerConfig(mixers[i % 3], ff) for i in range(layers)))


# Topapel at the same two widths, depths, vocabularies, attention head shapes and feed-forward widths
SHAPES.update({
    "topapel-tiny": _topapel_shape(64, 512, 3, 4, 2, 16, 24, 80, 2, 32, 128),
    "topapel-2k": _topapel_shape(2048, 32768, 8, 32, 8, 64, 1024, 2048, 16, 128, 8192),
    "topapel-4k": _topapel_shape(4096, 32768, 4, 32, 8, 128, 1024, 4096, 32, 128, 14336),
})


def _befirax_shape(width: int, vocab: int, layers: int, streams: int, heads: int, kv_heads: int, dim: int, vdim: int,
                   lat_heads: int, window: int, ssm_heads: int, experts: int, identity: int, top: int, expert_ff: int):
    """A Befirax shape at the sizes of a real model's layers: in turn a differential attention (`heads` on `kv_heads` heads of
    two maps of `dim`, half of whose dims are rotated, values of `vdim`, four taps), a latent attention (`lat_heads` heads of
    64 + 32 rotated dims over a latent of 96: a cache row as wide as the matrix-core attention's widest head; a window), a
    state-space layer (inner width twice the model's: `ssm_heads` heads of 64, state 128, four taps) and a differential
    attention on the keys and values of the first, each with routed experts some of which are the identity; `streams` copies
    of the residual stream."""
    from .config.befirax import (BefiraxConfig, BefiraxLayerConfig, DifferentialAttentionConfig, IdentityMoeConfig, PlainRotConfig,
                                 WindowedLatentConfig)
    from .config.kotipel import StateSpaceMixerConfig
    rot = PlainRotConfig(500000.0, dim // 2)
    moe = IdentityMoeConfig(experts, identity, top, expert_ff)
    out = []
    for i in range(layers):
        mixer = (DifferentialAttentionConfig(heads, kv_heads, dim, vdim, dim ** -0.5, 0.5, 4, rot),
                 WindowedLatentConfig(lat_heads, 64, 32, 64, 96, 96 ** -0.5, PlainRotConfig(1.0e6, 32), window),
                 StateSpaceMixerConfig(ssm_heads, 64, 128, 1, 4, 1),
                 DifferentialAttentionConfig(heads, kv_heads, dim, vdim, dim ** -0.5, 0.6, 4, rot, i - 3))[i % 4]
        out.append(BefiraxLayerConfig(mixer, moe))
    return BefiraxConfig(vocab=vocab, width=width, eps=1e-5, streams=streams, layers=tuple(out))


# Befirax at the same two widths, depths and vocabularies; its attention has as many query, key and value columns as the
# Llama shapes' (two maps of 64 and values of 128 where they have heads), its experts are Zozosun's and Timopel's
SHAPES.update({
    "befirax-tiny": _befirax_shape(64, 512, 4, 2, 2, 1, 16, 32, 2, 24, 2, 4, 2, 2, 32),
    "befirax-2k": _befirax_shape(2048, 32768, 8, 4, 16, 4, 64, 128, 16, 1024, 64, 32, 8, 4, 1024),
    "befirax-4k": _befirax_shape(4096, 32768, 4, 4, 32, 8, 64, 128, 32, 1024, 128, 64, 16, 6, 1536),
})
DESIGN_PAIRS = (("zozosun-2k", "llama-2k"), ("zozosun-4k", "llama-4k"), ("timopel-2k", "llama-2k"),
                ("timopel-4k", "llama-4k"), ("kotipel-2k", "llama-2k"), ("kotipel-4k", "llama-4k"),
                ("robuvik-2k", "llama-2k"), ("robuvik-4k", "llama-4k"), ("topapel-2k", "llama-2k"),
                ("topapel-4k", "llama-4k"), ("befirax-2k", "llama-2k"), ("befirax-4k", "llama-4k"))


def generate_requests(input_length: int, output_length: int, num_sequences: int, vocab_size: int,
                      fixed_lengths: bool = False, seed: int = 1352, min_input_length: int = 1,
                      fixed_output_length: bool = False):
    """serve/benchmark.py:12-24: lengths uniform in 1..input_length / 1..output_length, ids below
    10000, seed 1352.  `min_input_length` raises the lower end of the prompt lengths,
    `fixed_output_length` gives every request exactly `output_length` new tokens."""
    from .engine.engine import Request
    random.seed(seed)
    torch.manual_seed(seed)
    reqs = []
    for _ in range(num_sequences):
        n_in = input_length if fixed_lengths else random.randint(min_input_length, input_length)
        n_out = output_length if fixed_lengths or fixed_output_length else random.randint(1, output_length)
        ids = torch.randint(0, min(10000, vocab_size), (n_in,), dtype=torch.long)
        reqs.append(Request(input_ids=ids, input_length=n_in, max_new_tokens=n_out))
    return reqs


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="python -m serve_amd.benchmark", description=__doc__,
                                 formatter_class=argparse.RawDescriptionHelpFormatter)
    ap.add_argument("--profile", action="store_true", help="after the timed run, run once more under the profiler "
                    "and write a Chrome trace to /tmp/traces (serve/benchmark.py:82-101)")
    ap.add_argument("--profile-only", action="store_true", help="skip the timed run (serve/benchmark.py:69)")
    src = ap.add_mutually_exclusive_group()
    src.add_argument("--model", help="model folder (config.json + model.safetensors)")
    src.add_argument("--shape", "--preset", dest="shape", choices=sorted(SHAPES), default="llama-1b",
                     help="named shape, random weights")
    ap.add_argument("--dtype", type=lambda t: {"bf16": "bfloat16", "fp32": "float32"}.get(t, t),
                    choices=["bfloat16", "float32"], default="bfloat16", help="bfloat16 (or bf16), float32 (or fp32)")
    ap.add_argument("--input-length", type=int, default=256)
    ap.add_argument("--output-length", type=int, default=256)
    ap.add_argument("--num-sequences", type=int, default=2000)
    ap.add_argument("--temperature", type=float, default=0.6)
    ap.add_argument("--fixed-lengths", action="store_true", help="every request has exactly the given lengths")
    ap.add_argument("--min-input-length", type=int, default=1, help="prompt lengths are uniform from here to --input-length")
    ap.add_argument("--fixed-output-length", action="store_true", help="every request generates exactly --output-length tokens")
    ap.add_argument("--seed", type=int, default=0, help="seed of the random weights and of the sampler")
    ap.add_argument("--page-size", type=int, default=16)
    ap.add_argument("--memory-fraction", type=float, default=0.6, help="share of free memory for the cache "
                    "(serve/model.py:172)")
    ap.add_argument("--max-context", type=int, default=2048, help="serve/model.py:32")
    ap.add_argument("--max-requests", type=int, default=2048, help="requests live at a time at most; the reference "
                    "admits by cache capacity alone (serve/run.py:267-280)")
    ap.add_argument("--max-tokens-per-step", type=int, default=None,
                    help="tokens of a step, single decoded tokens and prompt portions together; default: 2048 + "
                         "--max-requests, since the reference prefills up to 2,048 prompt tokens a step "
                         "(serve/run.py:265) beside decode steps of their own")
    ap.add_argument("--prefill-chunk", type=int, default=2048)
    ap.add_argument("--admission", choices=["reserve", "optimistic"], default="reserve")
    ap.add_argument("--mixed-graphs", action="store_true", help="replay steps that carry prompt portions from graphs of "
                    "their padded shapes instead of launching them kernel by kernel: for small models with many live "
                    "requests, where the host is the bound")
    ap.add_argument("--phases", action="store_true", help="time the host's phases of the timed run (schedule, "
                    "plan_step, stage_copy, launch, read_back, ...) with named ranges and print their totals; the "
                    "ranges are also roctx markers for `rocprofv3 --marker-trace`")
    ap.add_argument("--admit-interval", type=int, default=1, help="admit new requests at most every N steps while "
                    "others run, so that the steps between are pure decode steps (1: at every step)")
    args = ap.parse_args(argv)

    from .engine.engine import Engine
    cfg = EngineConfig(dtype=args.dtype, page_size=args.page_size, memory_fraction=args.memory_fraction,
                       max_context=args.max_context, max_requests=args.max_requests,
                       max_tokens_per_step=args.max_tokens_per_step or 2048 + args.max_requests,
                       prefill_chunk=args.prefill_chunk,
                       admission=args.admission, admit_interval=args.admit_interval, seed=args.seed,
                       graph_mixed_steps=args.mixed_graphs)
    print(f"loading {args.model or args.shape} ({args.dtype}) ...", flush=True)
    if args.model:
        engine = Engine.from_folder(args.model, cfg)
    else:
        engine = Engine.from_config(SHAPES[args.shape], args.seed, cfg)
    print(f"model on the device; cache: {engine.runner.num_pages} pages of {args.page_size} tokens per group")
    requests = generate_requests(args.input_length, args.output_length, args.num_sequences,
                                 engine.model.spec.vocab_size, args.fixed_lengths,
                                 min_input_length=args.min_input_length, fixed_output_length=args.fixed_output_length)

    def fn():
        return engine.generate(requests, args.temperature)

    print(f"first run of {len(requests)} requests (loads the kernels, captures the graphs) ...", flush=True)
    st = time.perf_counter()
    fn()
    torch.cuda.synchronize()
    print(f"first run: {time.perf_counter() - st:.4f} s")
    if not args.profile_only:
        from . import trace
        if args.phases:
            trace.enable()
            trace.reset()
        torch.cuda.synchronize()
        st = time.perf_counter()
        responses = fn()
        torch.cuda.synchronize()
        elapsed = time.perf_counter() - st
        if args.phases:
            trace.disable()
        total = sum(len(r.generated_tokens) for r in responses)
        failed = [(i, r.error) for i, r in enumerate(responses) if r.error]
        if failed:
            print(f"{len(failed)} requests did not run; the first: request {failed[0][0]}: {failed[0][1]}",
                  file=sys.stderr)
            return 1
        print(f"timed run: {elapsed:.4f} s for {total} generated tokens")
        print(f"generated tokens per second: {total / elapsed:.2f}")
        if args.phases:
            print("host time inside the named ranges of the timed run (ranges nest: launch holds write_to_cache "
                  "and attention):")
            print(trace.report(elapsed))
    if args.profile or args.profile_only:
        import os
        name = f"generate_{args.input_length}_{args.output_length}_{args.num_sequences}"
        from . import trace
        trace.enable(markers=False, torch_ranges=True)
        with torch.profiler.profile() as prof:
            with torch.autograd.profiler.record_function(name):
                fn()
        trace.disable()
        os.makedirs("/tmp/traces", exist_ok=True)
        path = f"/tmp/traces/trace_{name}_{time.strftime('%H%M')}.json"
        prof.export_chrome_trace(path)
        print(f"profiler trace written to {path}")
    return 0


if __name__ == "__main__":
    sys.exit(main())
