"""A model as data: which parts make each layer, in which order layers run, whose cache a layer
reads.  ``Model`` builds the parts named by a ``ModelPlan`` from the part registry, collects their
declared weights and cache needs, and runs the layer list over a batch.

Reference shape of the same thing: ullm/models/qwen3.py:199-286 (embedding, layer loop carrying
(hidden, residual), final norm, lm_head on selected rows ullm/core/model_runner.py:339-341).
"""
from __future__ import annotations

from dataclasses import dataclass, field, replace
from typing import Any, Dict, List, Optional, Sequence, Tuple

import torch

from ..cache.manager import CacheGroupSpec
from ..kernels import ops
from ..parts import (Block, KVNeed, LayerCache, Norm, Part, PartEnv, StateNeed, StepContext, WeightDecl,
                     build_part, cache_needs_of, walk)
from ..parts.block import join_streams
from ..parts.linear import linear


EMBEDDER_CACHE = -1       # the cache id under which an embedder's per-request state is kept


@dataclass(frozen=True)
class Choice:
    """A part chosen by name with its parameters; parameters may themselves be choices."""
    kind: str
    name: str
    params: Dict[str, Any] = field(default_factory=dict)

    def build(self) -> Part:
        built = {k: (v.build() if isinstance(v, Choice) else v) for k, v in self.params.items()}
        return build_part(self.kind, self.name, **built)


@dataclass
class ModelPlan:
    vocab_size: int
    hidden_size: int
    embedding_weight: str                    # tensor name of the token table [vocab, hidden]
    layers: List[Choice]                     # one "block" choice per layer
    final_norm: Choice
    head_weight: str                         # tensor name of the output matrix [vocab, hidden]
    tie_head_to_embedding: bool = False      # bind the token table where the head tensor is absent
    embedding_scale: float = 1.0             # the token rows are multiplied by this on their way into the stream
    head_bias: Optional[str] = None          # tensor name of a bias [vocab] on the logits, float32
    logit_softcap: float = 0.0               # > 0: logits = cap * tanh(logits / cap)
    logit_scale: float = 1.0                 # the logits are multiplied by this
    # > 0: the residual stream is kept in this many copies (float32 [streams, T, hidden]), all equal to the embedding
    # output at the start; the layers' blocks read and write them, and the last norm is applied to their sum
    streams: int = 0
    # An "embedding" part that makes the stream's first rows (several tables, state of its own); it then owns the
    # token table and ``embedding_weight`` only names it (for a tied head).  None: the plain scaled row gather.
    embedder: Optional[Choice] = None
    # The order layers run in: (layer, cache id).  A layer may appear more than once (with a cache id
    # of its own each time, or the same one).  The first entry that names a cache id owns that cache
    # and writes it; later entries with the same id only read it, so a layer can read the cache
    # another layer wrote.  Default: every layer once, cache id = layer index.
    run_order: Optional[List[Tuple[int, int]]] = None
    # {cache id: cache id}: the layer that owns the first reads the paged caches of the second, written by a layer that
    # runs before it, in place of paged caches of its own; what it keeps beside those (fixed-size state) is its own.
    # The pages live as long as the widest window of the writer and all such readers asks for.
    kv_from: Dict[int, int] = field(default_factory=dict)
    # names a checkpoint may hold although this configuration has no use for them (a layer without a feed-forward
    # whose export still wrote that sublayer's norm): not loaded, and no error
    unused_tensors: Tuple[str, ...] = ()
    init_std: float = 0.02                   # random-weights mode

    def order(self) -> List[Tuple[int, int]]:
        return self.run_order if self.run_order is not None else [(i, i) for i in range(len(self.layers))]


class Model:
    def __init__(self, plan: ModelPlan):
        self.plan = plan
        self.blocks: List[Block] = [c.build() for c in plan.layers]
        self.final_norm: Norm = plan.final_norm.build()
        self.embedder = plan.embedder.build() if plan.embedder is not None else None
        self.run_order = plan.order()
        self.cache_owner: Dict[int, int] = {}      # cache id -> index into run_order of its owner
        for idx, (layer, cache_id) in enumerate(self.run_order):
            if not (0 <= layer < len(self.blocks)):
                raise ValueError(f"run order names layer {layer}: out of range")
            self.cache_owner.setdefault(cache_id, idx)
        for reader, source in plan.kv_from.items():
            if (reader not in self.cache_owner or source not in self.cache_owner or source in plan.kv_from
                    or self.cache_owner[source] >= self.cache_owner[reader]):
                raise ValueError(f"cache {reader} reads the keys of cache {source}: no layer with keys of its own that runs before it")
        self._keeps_embedding = any(b.needs_embedding for b in self.blocks)
        self.embedding: Optional[torch.Tensor] = None
        self.head: Optional[torch.Tensor] = None
        self.head_bias: Optional[torch.Tensor] = None
        self.env: Optional[PartEnv] = None

    # ------------------------------------------------------------------ weights
    def parts(self):
        if self.embedder is not None:
            yield from walk(self.embedder)
        for b in self.blocks:
            yield from walk(b)
        yield from walk(self.final_norm)

    def weight_decls(self) -> List[WeightDecl]:
        p = self.plan
        decls = [] if self.embedder is not None else [WeightDecl(p.embedding_weight, (p.vocab_size, p.hidden_size))]
        for part in self.parts():
            decls.extend(part.weights())
        decls.append(WeightDecl(p.head_weight, (p.vocab_size, p.hidden_size),
                                alias_of=p.embedding_weight if p.tie_head_to_embedding else None))
        if p.head_bias:
            decls.append(WeightDecl(p.head_bias, (p.vocab_size,), keep_fp32=True))
        return decls

    def bind(self, tensors: Dict[str, torch.Tensor], env: PartEnv) -> None:
        self.env = env
        self.embedding = tensors[self.plan.embedding_weight].contiguous()
        self.head = tensors[self.plan.head_weight].contiguous()
        self.head_bias = tensors[self.plan.head_bias].contiguous() if self.plan.head_bias else None
        for part in self.parts():
            part.bind(tensors, env)

    # ------------------------------------------------------------------ cache layout
    def cache_layout(self):
        """Groups of caches with equal needs, and the per-request state needs.  A cache is named by
        (cache id, index of the need among those its block declares).
        Returns (groups, {(cache id, need index): group index}, {(cache id, need index): StateNeed})."""
        keyed: Dict[KVNeed, List[Tuple[int, int]]] = {}
        states: Dict[Tuple[int, int], StateNeed] = {}
        if self.embedder is not None and self.embedder.cache_need() is not None:
            need = self.embedder.cache_need()
            if not isinstance(need, StateNeed):
                raise TypeError("an embedder keeps fixed-size state per request or nothing")
            states[(EMBEDDER_CACHE, 0)] = need
        own = {c: list(cache_needs_of(self.blocks[self.run_order[idx][0]])) for c, idx in self.cache_owner.items()}
        self._borrowed = {}
        for reader, source in self.plan.kv_from.items():
            mine = [i for i, n in enumerate(own[reader]) if isinstance(n, KVNeed)]
            theirs = [i for i, n in enumerate(own[source]) if isinstance(n, KVNeed)]
            if [replace(own[reader][i], window=0) for i in mine] != [replace(own[source][i], window=0) for i in theirs]:
                raise ValueError(f"cache {reader} reads the keys of cache {source} but their rows differ")
            for i, j in zip(mine, theirs):
                a, b = own[reader][i].window, own[source][j].window
                own[source][j] = replace(own[source][j], window=max(a, b) if a and b else 0)
                self._borrowed[(reader, i)] = (source, j)
        for cache_id, needs in own.items():
            for i, need in enumerate(needs):
                if (cache_id, i) in self._borrowed:
                    continue
                if isinstance(need, KVNeed):
                    keyed.setdefault(need, []).append((cache_id, i))
                else:
                    states[(cache_id, i)] = need
        groups, cache_group = [], {}
        for need, keys in keyed.items():
            for c in keys:
                cache_group[c] = len(groups)
            rows = tuple((r.heads, r.dim, None if r.dtype is None else torch.empty((), dtype=r.dtype).element_size())
                         for r in need.rows) if need.rows else None
            groups.append(CacheGroupSpec(need.num_kv_heads, need.head_dim, need.window, tuple(keys), rows,
                                         need.tokens_per_row, need.chunk))
        self._group_needs = list(keyed)
        for idx, (layer, cache_id) in enumerate(self.run_order):
            owner_layer = self.run_order[self.cache_owner[cache_id]][0]
            a, b = cache_needs_of(self.blocks[layer]), cache_needs_of(self.blocks[owner_layer])
            if a != b:
                raise ValueError(f"layer {layer} reads cache {cache_id} written by layer {owner_layer} "
                                 f"but their needs differ: {a} vs {b}")
        return groups, cache_group, states

    def group_needs(self) -> List[KVNeed]:
        """The paged need of every cache group, in the order of :meth:`cache_layout`'s groups."""
        self.cache_layout()
        return self._group_needs

    def borrowed_caches(self) -> Dict[Tuple[int, int], Tuple[int, int]]:
        """{(cache id, need index): (cache id, need index) of the cache it reads instead} (see ``ModelPlan.kv_from``)."""
        self.cache_layout()
        return self._borrowed

    def num_needs(self, cache_id: int) -> int:
        """How many needs the block that owns this cache declares."""
        if cache_id == EMBEDDER_CACHE:
            return 1
        return len(cache_needs_of(self.blocks[self.run_order[self.cache_owner[cache_id]][0]]))

    # ------------------------------------------------------------------ forward
    def forward(self, ctx: StepContext, caches: Dict[int, LayerCache], logit_rows: Optional[torch.Tensor]):
        """Runs the batch through every layer of the run order and returns float32 logits
        [len(logit_rows), vocab] (None if no row is wanted)."""
        if self.embedder is not None:
            residual = self.embedder.forward(ctx, caches.get(EMBEDDER_CACHE) or LayerCache())
        else:
            residual = ops.embedding(ctx.token_ids, self.embedding, scale=self.plan.embedding_scale)
        pending = None
        if self.plan.streams > 0:
            residual = ops.streams_spread(residual, self.plan.streams)
        if self._keeps_embedding:
            ctx.embedded = residual.clone()      # the stream's rows are written in place from here on
        for idx, (layer, cache_id) in enumerate(self.run_order):
            cache = caches.get(cache_id)
            if cache is None:
                cache = LayerCache()
            elif self.cache_owner[cache_id] != idx:
                cache = cache.reader()
            block = self.blocks[layer]
            if block.hands_norm_ahead and idx + 1 < len(self.run_order):
                # a block whose last kernel can prepare the norm that follows is told which norm that is
                after = self.blocks[self.run_order[idx + 1][0]].entry_norm()
                residual, pending = block.forward(residual, pending, ctx, cache, next_norm=after)
            else:
                residual, pending = block.forward(residual, pending, ctx, cache)
        if logit_rows is None or logit_rows.numel() == 0:
            return None
        if self.plan.streams > 0:
            x = join_streams(residual, pending, self.final_norm, logit_rows, ctx.dtype)
        else:
            x = self.final_norm.add_norm(pending, residual, rows=logit_rows, out_dtype=ctx.dtype)
        logits = linear(x, self.head, self.head_bias, out_dtype=torch.float32)
        if self.plan.logit_scale != 1.0:
            ops.scale_(logits, self.plan.logit_scale)
        if self.plan.logit_softcap > 0:
            ops.softcap_(logits, self.plan.logit_softcap)
        return logits
