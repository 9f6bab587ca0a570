"""`Befirax`: a decoder whose layers are listed one by one in config.json, as a `ModelSpec`.

The residual stream is several copies, which every sublayer reads as a weighted sum and writes back to through a matrix
(arrangement `hyper_residual`); the final norm takes their sum.  The mixer is "attention" (differential attention whose
queries, keys and values pass a short convolution, with an element-wise output gate, biases, and possibly another
layer's keys and values), "latent_attention" (one normed latent and one rotated key part per token for all heads, a
sliding window, a gate per head) or "mamba2" (the state-space mixer).  The feed-forward is absent or a mixture of experts
chosen by corrected shares of a softmax, some of which are the identity.  The output matrix is the embedding table.

Tensor names: `embed`, `l<i>.norm1|norm2`, `l<i>.hc1|hc2.in|out|mix`, `l<i>.mix.*`, `l<i>.mlp.*`, `final.norm`.
"""
from __future__ import annotations

from ..config.befirax import BefiraxConfig, DifferentialAttentionConfig, WindowedLatentConfig
from ..config.spec import LayerSpec, ModelSpec, PartSpec, RunEntry
from ..registry import register_architecture


def _position(rot, head_dim: int, pairing: str):
    if rot is None:
        return None
    # (undivided frequencies, from float64)
    return PartSpec("rope", {"head_dim": head_dim, "rot_dim": rot.dims, "theta": rot.base, "pairing": pairing,
                             "scaling": {"rope_type": "linear", "factor": 1.0}})


def _attention(m: DifferentialAttentionConfig, d: int, eps: float):
    own = m.kv_from is None
    part = PartSpec("differential_attention", {
        "hidden_size": d, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim, "scale": m.scale,
        "eps": eps, "diff": m.diff, "position": _position(m.rot, m.dim, "adjacent"), "conv": m.conv, "bias": True,
        "out_gate": True, "own_kv": own})
    names = ["lq1", "lk1", "lq2", "lk2", "g", "o", "o.b"]
    for n in ("q", "k", "v") if own else ("q",):
        names += [n, n + ".b"] + ([n + ".conv"] if m.conv else [])
    return part, names


def _latent(m: WindowedLatentConfig, d: int, eps: float):
    part = PartSpec("latent_attention", {
        "hidden_size": d, "heads": m.heads, "dim": m.dim, "rot_dim": m.rot_dim, "vdim": m.vdim, "kv_rank": m.kv_rank,
        "scale": m.scale, "eps": eps, "position": _position(m.rot, m.rot_dim, "half"), "window": m.window,
        "retain": m.window, "out_gate": "head"})
    return part, ["q", "dkv", "dkv.norm", "uk", "uv", "g", "o"]


def _state_space(m, d: int, eps: float):
    part = PartSpec("state_space", {"hidden_size": d, "heads": m.heads, "vdim": m.vdim, "state": m.state, "groups": m.groups,
                                    "conv": m.conv, "norm_groups": m.norm_groups, "eps": eps})
    return part, ["in", "conv", "conv.b", "dt_bias", "A_log", "D", "norm", "o"]


def build_befirax_spec(cfg: BefiraxConfig) -> ModelSpec:
    d, S = cfg.width, cfg.streams
    norm = PartSpec("rmsnorm", {"size": d, "eps": cfg.eps})
    streams = PartSpec("hyper_connection", {"streams": S})
    layers, run_order = [], []
    for i, layer in enumerate(cfg.layers):
        p, m, mlp = f"l{i}.", layer.mixer, layer.mlp
        build = (_attention if isinstance(m, DifferentialAttentionConfig)
                 else _latent if isinstance(m, WindowedLatentConfig) else _state_space)
        mixer, names = build(m, d, cfg.eps)
        parts = {"mixer": mixer, "mixer_norm": norm, "mixer_streams": streams}
        weights = {"mixer_norm.weight": p + "norm1"}
        weights.update({"mixer_streams." + n: p + "hc1." + n for n in ("in", "out", "mix")})
        weights.update({"mixer." + n: p + "mix." + n for n in names})
        if mlp is not None:
            parts.update(ffn_norm=norm, ffn_streams=streams, ffn=PartSpec("routed_experts", {
                "hidden_size": d, "experts": mlp.experts, "top": mlp.top, "expert_size": mlp.ff, "router_softmax": "all",
                "identity": mlp.identity, "correction": True}))
            weights["ffn_norm.weight"] = p + "norm2"
            weights.update({"ffn_streams." + n: p + "hc2." + n for n in ("in", "out", "mix")})
            names = ["router", "correction"] + [f"e{e}.{n}" for e in range(mlp.experts) for n in ("gate", "up", "down")]
            weights.update({"ffn." + n: p + "mlp." + n for n in names})
        layers.append(LayerSpec(parts=parts, weights=weights, arrangement="hyper_residual"))
        # every layer has a cache layer of its own, also where that holds no more than its state
        src = getattr(m, "kv_from", None)
        run_order.append(RunEntry(layer=i, cache=i, writes_cache=src is None, reads_pages_of=src))
    return ModelSpec(
        architecture=cfg.architecture, vocab_size=cfg.vocab, hidden_size=d,
        embedding=PartSpec("token_embedding", {"vocab_size": cfg.vocab, "hidden_size": d, "copies": S}),
        layers=layers, run_order=run_order,
        final_norm=PartSpec("merged_streams_rmsnorm", {"size": d, "eps": cfg.eps, "streams": S}),
        lm_head=PartSpec("linear_head", {"vocab_size": cfg.vocab, "hidden_size": d, "tied": True, "shares": "embedding.weight"}),
        weights={"embedding.weight": "embed", "final_norm.weight": "final.norm", "lm_head.weight": "embed"},
        # a layer without feed-forward may still carry the norm and the stream weights of one: nothing reads them
        ignored_weight_patterns=[r"l\d+\.norm2", r"l\d+\.hc2\.(in|out|mix)"],
    )


register_architecture("Befirax", BefiraxConfig.from_hf_dict, build_befirax_spec)
