"""`Topapel`: a decoder whose layers are listed one by one in config.json, as a `ModelSpec`.

A layer is pre-norm, x <- x + mixer(N_1(x)); x <- x + ff(N_2(x)) (the second half only if the layer has a feed-forward),
with norm weights stored around zero.  The mixer is "attention" (grouped-query attention with biases, queries and keys
normed per head, the un-normed keys as values, a rotation with divided frequencies, a learned sink per head, and a mask of
chunks of positions), "lightning" (a linear attention with one constant decay per head) or "mingru" (an element-wise gated
average).  The feed-forward's activation is a polynomial of normed powers.  The output matrix is the embedding table; its
logits are scaled and kept within a soft cap.

Tensor names: `embed`, `l<i>.norm1|norm2`, `l<i>.mix.*`, `l<i>.mlp.up|down|act`, `final.norm`.
"""
from __future__ import annotations

from ..config.spec import LayerSpec, ModelSpec, PartSpec, RunEntry
from ..config.topapel import ChunkAttentionConfig, LightningConfig, TopapelConfig
from ..registry import register_architecture


def _mixer(m, d: int, eps: float):
    """(the mixer's spec, its tensors' local names)"""
    if isinstance(m, ChunkAttentionConfig):
        position = None
        if m.rot is not None:
            scaling = None if m.rot.factor is None else {"rope_type": "linear", "factor": m.rot.factor}
            position = PartSpec("rope", {"head_dim": m.dim, "rot_dim": m.rot.dims, "theta": m.rot.base,
                                         "scaling": scaling, "pairing": "half"})
        return (PartSpec("qk_norm_attention", {
            "hidden_size": d, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.dim,
            "scale": m.scale, "eps": eps, "sink": True, "position": position, "bias": True, "out_bias": True,
            "values": "keys", "chunk": m.chunk}),
            ["q", "k", "q.b", "k.b", "q.norm", "k.norm", "sink", "o", "o.b"])
    if isinstance(m, LightningConfig):
        return (PartSpec("decayed_linear_attention", {"hidden_size": d, "heads": m.heads, "dim": m.dim, "vdim": m.vdim,
                                                      "decay": m.decay, "eps": eps}),
                ["q", "k", "v", "g", "o", "norm"])
    return (PartSpec("gated_average", {"hidden_size": d, "width": m.width}), ["z", "z.b", "x", "x.b", "g", "o"])


def build_topapel_spec(cfg: TopapelConfig) -> ModelSpec:
    d = cfg.width
    norm = PartSpec("rmsnorm", {"size": d, "eps": cfg.eps, "offset": 1.0})
    layers = []
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}."
        mixer, names = _mixer(layer.mixer, d, cfg.eps)
        parts = {"mixer": mixer, "mixer_norm": norm}
        weights = {"mixer_norm.weight": p + "norm1"}
        weights.update({"mixer." + n: p + "mix." + n for n in names})
        if layer.ff is not None:
            parts.update(ffn_norm=norm, ffn=PartSpec("dense", {"hidden_size": d, "intermediate_size": layer.ff,
                                                               "activation": "poly_norm", "eps": cfg.eps}))
            weights["ffn_norm.weight"] = p + "norm2"
            weights.update({"ffn." + n: p + "mlp." + n for n in ("up", "down", "act")})
        layers.append(LayerSpec(parts=parts, weights=weights, arrangement="prenorm_residual"))
    return ModelSpec(
        architecture=cfg.architecture, vocab_size=cfg.vocab, hidden_size=d,
        embedding=PartSpec("token_embedding", {"vocab_size": cfg.vocab, "hidden_size": d, "scale": cfg.embedding_scale}),
        layers=layers, run_order=[RunEntry(layer=i, cache=i) for i in range(len(layers))],
        final_norm=norm,
        lm_head=PartSpec("linear_head", {"vocab_size": cfg.vocab, "hidden_size": d, "tied": True,
                                         "shares": "embedding.weight", "scale": cfg.logit_scale,
                                         "soft_cap": cfg.logit_softcap}),
        weights={"embedding.weight": "embed", "final_norm.weight": "final.norm", "lm_head.weight": "embed"},
        # a layer without feed-forward may still carry the norm in front of one: nothing reads it
        ignored_weight_patterns=[r"l\d+\.norm2"],
    )


register_architecture("Topapel", TopapelConfig.from_hf_dict, build_topapel_spec)
