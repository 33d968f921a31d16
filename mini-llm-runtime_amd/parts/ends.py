"""The two ends of a decoder: the embedding that turns a step's token ids into the float residual stream
(src/minillm/runtime.cpp:224-228, src/minillm/cuda/runtime.cpp:184-188) and the output head that turns the
normed rows whose logits are wanted into logits (src/minillm/runtime.cpp:338-351).  Both are parts like any
other: built from a spec by its `kind`, asked for their tensors, their kernel libraries and their scratch
buffers, so that a model with a multiplier on its embedding, a cap on its logits or a bias on its head
registers another kind instead of editing the model."""
from __future__ import annotations

import torch

from ..cache.manager import StateSpec
from ..config.specs import EmbedSpec, HeadSpec
from ..weights.loader import WeightSpec
from .registry import PartError, register_part

__all__ = ["TokenEmbedding", "PairEmbedding", "RunVectors", "LinearHead", "ScaledHead", "CappedHead", "EmbedSpec", "HeadSpec"]


@register_part("embed", "token_embedding")
class TokenEmbedding:
    graph_safe = True        # forward launches kernels over the step's device vectors only

    def __init__(self, spec):
        if spec.vocab_size < 1 or spec.hidden < 1:
            raise PartError("an embedding needs a vocabulary and a width")
        self.spec = spec
        self.weight = None

    def weight_specs(self):
        return {"weight": WeightSpec((self.spec.vocab_size, self.spec.hidden))}

    def bind(self, weights):
        self.weight = weights["weight"]

    def libraries(self):
        return ["elementwise"]

    def workspace_plan(self, rows, logits_rows, dtype, limits):
        return {("hidden", torch.float32): rows * self.spec.hidden}

    def table(self):
        """The [vocab, hidden] matrix, for a head that is tied to it."""
        return self.weight

    def forward(self, ctx):
        """The float residual stream [B, E] of the step's tokens: the table's rows times the spec's factor."""
        h = ctx.workspace.get("hidden", (ctx.n_tokens, self.spec.hidden), torch.float32)
        ctx.kernels.embed_gather(ctx.token_ids, self.weight, h, float(getattr(self.spec, "scale", 1.0)))
        return h


@register_part("embed", "run_vectors")
class RunVectors:
    """Learned vectors that runs of the schedule add to the residual stream, one row of [count, hidden] each; 32-bit."""
    graph_safe = True

    def __init__(self, spec):
        if spec.count < 1 or spec.hidden < 1:
            raise PartError("run vectors need a count and a width")
        self.spec = spec
        self.weight = None

    def weight_specs(self):
        return {"weight": WeightSpec((self.spec.count, self.spec.hidden), keep_float32=True, init=("normal", 0.0, 0.3))}

    def bind(self, weights):
        self.weight = weights["weight"]

    def libraries(self):
        return ["elementwise"]

    def row(self, i):
        return self.weight[i]


@register_part("embed", "pair_embedding")
class PairEmbedding(TokenEmbedding):
    """A token's embedding plus a row of a second table that the token and the one before it pick:
    row (previous * mul_prev + token * mul_cur) mod buckets, and the table's last row (number `buckets`) for a
    request's first token.  The token before a step's first token of a request is state of the request: an embedding
    with a `cache_spec()` gets a cache entry like a mixer does (`cache_id`, set by the model), here one integer a
    slot, staged by the last row a request brings and made live with every other state when the step has run."""
    graph_safe = True

    def __init__(self, spec):
        super().__init__(spec)
        if spec.buckets < 1:
            raise PartError("the pair table needs at least one bucket")
        self.pairs = None
        self.cache_id = None

    def weight_specs(self):
        s = self.spec
        return {"weight": WeightSpec((s.vocab_size, s.hidden)), "pairs": WeightSpec((s.buckets + 1, s.hidden))}

    def bind(self, weights):
        self.weight, self.pairs = weights["weight"], weights["pairs"]

    def cache_spec(self):
        return StateSpec((1,), torch.int32)

    def forward(self, ctx):
        s = self.spec
        h = ctx.workspace.get("hidden", (ctx.n_tokens, s.hidden), torch.float32)
        ctx.kernels.pair_embed(ctx.token_ids, ctx.positions, ctx.slots, self.weight, self.pairs,
                               ctx.cache.state_view(self.cache_id), ctx.cache.state_stage(self.cache_id), h,
                               s.buckets, s.mul_prev % s.buckets, s.mul_cur % s.buckets)     # (the same rows; the kernel's
        return h                                                                                    # products stay small)


@register_part("head", "linear_head")
class LinearHead:
    graph_safe = True

    def __init__(self, spec):
        self.spec = spec
        self.weight = None

    def weight_specs(self):
        # (a tied head has no tensor of its own; a file that carries one anyway is taken at its word)
        return {"weight": WeightSpec((self.spec.vocab_size, self.spec.hidden), optional=self.spec.tied)}

    def bind(self, weights, embed=None):
        """`embed`: the model's embedding part; a tied head without a tensor of its own takes its table (the
        same memory, no copy)."""
        if "weight" in weights:
            self.weight = weights["weight"]
        elif self.spec.tied and embed is not None and hasattr(embed, "table"):
            self.weight = embed.table()
        else:
            raise PartError("the output head has no weight and nothing to be tied to")

    def libraries(self):
        return ["gemm"]

    def workspace_plan(self, rows, logits_rows, dtype, limits):
        return {("logits", torch.float32): logits_rows * self.spec.vocab_size}

    def forward(self, ctx, final):
        """float logits [R, V] of the normed rows `final` [R, E]."""
        logits = ctx.workspace.get("logits", (final.shape[0], self.spec.vocab_size), torch.float32)
        ctx.kernels.gemm(final, self.weight, logits)
        return logits


@register_part("head", "scaled_head")
class ScaledHead(LinearHead):
    """logits = (final . weight^T) * scale, the factor applied to the 32-bit logits."""

    def libraries(self):
        return ["gemm", "elementwise"]

    def forward(self, ctx, final):
        logits = super().forward(ctx, final)
        if self.spec.scale != 1.0:
            ctx.kernels.scale_float(logits, float(self.spec.scale))
        return logits


@register_part("head", "capped_head")
class CappedHead(LinearHead):
    """logits <- softcap * tanh(logits / softcap) on the 32-bit logits (no cap: a plain head)."""

    def libraries(self):
        return ["gemm", "elementwise"]

    def forward(self, ctx, final):
        logits = super().forward(ctx, final)
        if self.spec.softcap is not None:
            ctx.kernels.tanh_cap(logits, float(self.spec.softcap))
        return logits
