"""The generic model: a `ModelSpec` built into parts, with the list of tensors it needs and
one forward pass over the tokens of a step (serve/model.py:196-231 without the
prefill/decode split: the same code runs prompt portions and single tokens).
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, List, Optional, Tuple

import torch

from ..cache.retention import Retention
from ..config.spec import ModelSpec, PartSpec
from ..parts.base import LayerCache, Part, Runtime, StateRequest, TokenCacheRequest
from ..registry import get_part


@dataclass(frozen=True)
class WeightRequest:
    """A checkpoint tensor the model needs: where it comes from and where it goes."""

    checkpoint_name: str
    owner: str            # "layers.3.mixer", "embedding", ...
    local_name: str       # the part's own name for it
    shape: Tuple[int, ...]
    init: str
    optional: bool
    alias_of: Optional[str] = None     # "owner.local_name" of the tensor that serves in its place
    alias_only: bool = False           # the checkpoint's own copy is never read


def _make(role: str, spec: PartSpec):
    return get_part(role, spec.kind)(**spec.params)


class Model:
    def __init__(self, spec: ModelSpec):
        self.spec = spec
        self.embedding = _make("embedding", spec.embedding)
        self.final_norm = _make("norm", spec.final_norm)
        self.lm_head = _make("lm_head", spec.lm_head)
        self.pass_vectors = None if spec.pass_vectors is None else _make("stream_input", spec.pass_vectors)
        self.layers = []
        for i, ls in enumerate(spec.layers):
            arrangement = get_part("arrangement", ls.arrangement)
            roles = arrangement.PART_ROLES              # part name -> registry role
            optional = set(getattr(arrangement, "OPTIONAL_PARTS", ()))      # (a layer without a feed-forward)
            if not (set(roles) - optional) <= set(ls.parts) <= set(roles):
                raise ValueError(f"layer {i}: arrangement {ls.arrangement!r} is built from the parts "
                                 f"{sorted(roles)}, the spec gives {sorted(ls.parts)}")
            layer = arrangement(**{name: _make(roles[name], ps) for name, ps in ls.parts.items()})
            biased = [n for n, p in layer.parts().items() if getattr(p, "has_output_bias", False)]
            if biased and not getattr(arrangement, "adds_output_bias", False):
                raise ValueError(f"layer {i}: arrangement {ls.arrangement!r} does not add the output bias of {biased}")
            self.layers.append(layer)
        for e in spec.run_order:
            if not 0 <= e.layer < len(self.layers):
                raise ValueError(f"run order names layer {e.layer}, the model has {len(self.layers)}")
            if e.pass_vector is not None and self.pass_vectors is None:
                raise ValueError("the run order names a pass vector, the model has no table of them")
            if e.adds_embedding and e.pass_vector is None:
                raise ValueError("the embedding's output is added again together with a pass vector")
        self._check_cache_owners()
        self.rt: Optional[Runtime] = None

    # -- what the model needs ---------------------------------------------------------------
    def _owners(self) -> Dict[str, Part]:
        owners: Dict[str, Part] = {"embedding": self.embedding, "final_norm": self.final_norm,
                                   "lm_head": self.lm_head}
        if self.pass_vectors is not None:
            owners["pass_vectors"] = self.pass_vectors
        for i, layer in enumerate(self.layers):
            for name, part in layer.parts().items():
                owners[f"layers.{i}.{name}"] = part
        return owners

    def weight_requests(self) -> List[WeightRequest]:
        out: List[WeightRequest] = []

        def add(owner: str, part: Part, names: Dict[str, str], prefix: str):
            for pr in part.param_requests():
                key = prefix + pr.name
                if key not in names:
                    raise KeyError(f"the spec gives no checkpoint name for {owner}.{pr.name}")
                out.append(WeightRequest(names[key], owner, pr.name, tuple(pr.shape), pr.init, pr.optional,
                                         pr.alias_of, pr.alias_only))

        add("embedding", self.embedding, self.spec.weights, "embedding.")
        if self.pass_vectors is not None:
            add("pass_vectors", self.pass_vectors, self.spec.weights, "pass_vectors.")
        for i, (layer, ls) in enumerate(zip(self.layers, self.spec.layers)):
            for name, part in layer.parts().items():
                add(f"layers.{i}.{name}", part, ls.weights, name + ".")
        add("final_norm", self.final_norm, self.spec.weights, "final_norm.")
        add("lm_head", self.lm_head, self.spec.weights, "lm_head.")
        return out

    def _check_cache_owners(self) -> None:
        writers: Dict[int, int] = {}
        for e in self.spec.run_order:
            if e.reads_pages_of is not None and e.writes_cache:
                raise ValueError("an entry of the run order that reads another cache layer's pages does not write them")
            if e.writes_cache or e.reads_pages_of is not None:
                if e.cache in writers:
                    raise ValueError(f"cache layer {e.cache} is written by two entries of the run order")
                writers[e.cache] = e.layer
        n = self.spec.num_cache_layers()
        for c in range(n):
            if c not in writers:
                raise ValueError(f"cache layer {c} is read but never written")
        self._cache_writer_layer = [writers[c] for c in range(n)]
        written = set()
        for e in self.spec.run_order:
            if e.reads_pages_of is not None and e.reads_pages_of not in written:
                raise ValueError(f"cache layer {e.reads_pages_of} is read before anything has written it")
            if e.writes_cache:
                written.add(e.cache)
            elif e.reads_pages_of is not None and self._cache_owner(e.layer).cache_request() is not None:
                raise ValueError(f"layer {e.layer} keeps keys of its own and cannot read another layer's")

    def _cache_owner(self, layer: int) -> Optional[Part]:
        return self.layers[layer].cache_owner()

    def _embedding_state(self) -> Optional[StateRequest]:
        """Per-request state of the embedding (a part that looks back at a request's earlier tokens), or None."""
        return self.embedding.state_request() if hasattr(self.embedding, "state_request") else None

    def cache_requests(self) -> List[Optional[TokenCacheRequest]]:
        """Per cache layer: what the part that writes it keeps per token.  An embedding with per-request state
        has one more cache layer, the last, that holds nothing per token."""
        owners = [self._cache_owner(l) for l in self._cache_writer_layer]
        out = [None if o is None else o.cache_request() for o in owners]
        return out + [None] if self._embedding_state() is not None else out

    def state_requests(self) -> List[Optional[StateRequest]]:
        """Per cache layer: the fixed-size per-request state its part needs (the embedding's, if it has one, in a
        last cache layer of its own)."""
        owners = [self._cache_owner(l) for l in self._cache_writer_layer]
        out = [None if o is None else o.state_request() for o in owners]
        emb = self._embedding_state()
        return out + [emb] if emb is not None else out

    # -- what a step costs (for measurements) ---------------------------------------------------
    def step_cost(self, tokens: int, logit_rows: int = 1, context_before: int = 0):
        """(elements of weights read, flops) of a step that runs `tokens` tokens of one request with
        `context_before` tokens in the cache and computes `logit_rows` rows of logits: the parts'
        own accounts (`Part.step_cost`) added up along the run order, so that a layer that runs
        twice is read and computed twice.  Norms and the embedding's gathered rows count as their
        parts say (the framework's: their weights, and nothing)."""
        elements, flops = 0, 0.0
        emb = self.embedding.step_cost(tokens, context_before)
        elements, flops = elements + emb.weight_elements, flops + emb.flops
        for e in self.spec.run_order:
            for part in self.layers[e.layer].parts().values():
                c = part.step_cost(tokens, context_before)
                elements, flops = elements + c.weight_elements, flops + c.flops
        for part, n in ((self.final_norm, logit_rows), (self.lm_head, logit_rows)):
            c = part.step_cost(n, 0)
            elements, flops = elements + c.weight_elements, flops + c.flops
        return elements, flops

    def cache_elements_per_token(self) -> List[Tuple[int, Retention]]:
        """Per cache layer that is read in a step (once per run-order entry that works on it):
        (elements kept per token, retention rule)."""
        reqs = self.cache_requests()
        out = []
        for e in self.spec.run_order:
            r = reqs[e.cache if e.reads_pages_of is None else e.reads_pages_of]
            if r is not None:
                out.append((sum(t.elements_per_token() for t in r.tensors), r.retention))
        return out

    def graph_safe(self) -> bool:
        """Whether every part only enqueues GPU work, so that a step can be captured into a graph."""
        return all(getattr(p, "graph_safe", False) for p in self._owners().values())

    # -- loading ------------------------------------------------------------------------------
    def load(self, tensors_by_owner: Dict[str, Dict[str, torch.Tensor]], rt: Runtime) -> None:
        """Hand every part its tensors.  A request with `alias_of` that got no tensor of its own
        receives the named tensor of the other part: the same device memory, no copy."""
        self.rt = rt
        given = {owner: dict(t) for owner, t in tensors_by_owner.items()}
        for r in self.weight_requests():
            if r.alias_of is None or r.local_name in given.get(r.owner, {}):
                continue
            other = max((o for o in self._owners() if r.alias_of.startswith(o + ".")), key=len, default="")
            local = r.alias_of[len(other) + 1:]
            if local not in given.get(other, {}):
                raise KeyError(f"{r.owner}.{r.local_name} stands for {r.alias_of}, which was not loaded")
            t = given[other][local]
            if tuple(t.shape) != tuple(r.shape):
                raise ValueError(f"{r.owner}.{r.local_name} {list(r.shape)} cannot share {r.alias_of} {list(t.shape)}")
            given.setdefault(r.owner, {})[r.local_name] = t
        for owner, part in self._owners().items():
            part.load(given.get(owner, {}), rt)

    # -- running -------------------------------------------------------------------------------
    def forward(self, ctx, caches: List[LayerCache]) -> torch.Tensor:
        """Run the tokens of one step; return fp32 logits [R, V] at ctx.logit_rows."""
        again = any(e.adds_embedding for e in self.spec.run_order)
        x0 = None
        if self._embedding_state() is not None:
            # (its state lies in the cache layer behind the run order's)
            x = self.embedding.forward(ctx, caches[self.spec.num_cache_layers()], keep=again)
            if again:
                x, x0 = x
        else:
            x = self.embedding.forward(ctx)
            if again:
                x0 = x.clone()
        ctx.stream_copy = None          # (what a layer may leave for the next: the stream in the activation dtype)
        ctx.shared = {}                 # (and what layers leave for later layers of the step, by name)
        pending = None
        order = self.spec.run_order
        for i, e in enumerate(order):
            # the norm the next layer begins with, where its arrangement says so: this layer may apply it at the
            # end of its own last kernel and leave the result in ctx.shared
            nxt = self.layers[order[i + 1].layer] if i + 1 < len(order) else None
            ctx.next_input_norm = nxt.input_norm() if hasattr(nxt, "input_norm") else None
            if nxt is not None and order[i + 1].pass_vector is not None:
                ctx.next_input_norm = None          # (the stream changes between the two layers)
            if e.pass_vector is not None:
                pending = self.pass_vectors.forward(x, pending, e.pass_vector, x0 if e.adds_embedding else None)
            cache = caches[e.cache]
            if e.reads_pages_of is not None:
                cache = caches[e.reads_pages_of].with_state_of(cache)
            pending = self.layers[e.layer].forward(x, pending, ctx, cache, e.writes_cache)
        if ctx.num_logit_rows == 0:
            return torch.empty((0, self.spec.vocab_size), dtype=torch.float32, device=x.device)
        h = self.final_norm.forward(x, pending, rows=ctx.logit_rows)
        out = getattr(ctx, "logits_out", None)
        if out is not None and getattr(self.lm_head, "accepts_out", False):
            return self.lm_head.forward(h, out=out)        # the caller's buffer (a replayed step's fixed one)
        return self.lm_head.forward(h)
