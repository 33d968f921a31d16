"""Causal grouped-query attention whose heads look at each other between the softmax and the values: head h's weights
become sum_g mix[h, g] weights_g before they meet the values of h's own kv head.  Around it, each optional: a norm
per head of q and k before their rotation (a head's first channels, as the position part says), a cap on the scores, a
sink in the softmax (a constant or a number a head), VALUES turned by their position before they are cached -- every
head's output is turned back by the query's position --, and one sigmoid gate a head.

Per token the cache keeps the turned keys [kv_heads, head_dim] and the turned values [kv_heads, value_dim], the values
transposed within a page.

The bfloat16 engine runs the attention on the matrix cores where they take the sizes (`Kernels.head_mix_tiles`: the
exponentials of all scores go through scratch memory, bounded by taking a step's tokens in portions); else, and in the
float engine, one workgroup a token, whose sums follow from the token's position alone.
"""
from __future__ import annotations

import torch

from ..cache.manager import PAGE, PagedSpec
from ..weights.loader import WeightSpec, stacked
from .registry import PartError, build_part, register_part
from .sink_attention import _rope_table

GROUP = 16                    # tokens of a group of a prompt portion (single tokens: groups of one)
SCRATCH_CAP = 144 << 20       # elements of exponentials that one launch may keep at most (one group may take more)
PARTIAL_CAP = 16 << 20        # floats of the key ranges' shares
SUMS_CAP = 4 << 20            # floats of the sums
MOST_RANGES = 64
RANGE = 256                   # the narrowest range of keys of a workgroup
WIDE_RANGE = 1024             # and the one that costs nothing


def _up(n, unit):
    return -(-n // unit) * unit


class LaunchShape:
    """How `groups` groups of `tokens` tokens over contexts up to `context` keys are launched."""

    def __init__(self, spec, layout, groups, tokens, context, target):
        pad, inner, most = layout
        s = spec
        self.ktiles = -(-context // 32)
        keys = self.ktiles * 32
        row_e, row_o = keys * inner, s.q_heads * s.value_dim
        # groups a launch: what the scratch buffers hold (at least one)
        self.groups = max(1, min(groups, SCRATCH_CAP // (tokens * row_e), PARTIAL_CAP // (tokens * row_o),
                                 SUMS_CAP // (tokens * inner)))
        # ranges of keys where the groups alone do not fill the GPU
        tiles = -(-tokens * pad // 16)
        units = self.groups * (inner // pad) * -(-tiles // (4 if tiles >= 4 else 2 if tiles >= 2 else 1))
        ranges = max(1, min(MOST_RANGES, -(-target // units), keys // RANGE, SUMS_CAP // (self.groups * tokens * inner)))
        self.score_keys = _up(-(-keys // ranges), 128)
        self.score_ranges = -(-keys // self.score_keys)
        # the second launch: wide ranges first, then fewer kv heads a workgroup (each mixes for its own), then narrow
        # ranges (their shares are written and read again), measured in this order
        room = max(1, PARTIAL_CAP // (self.groups * tokens * row_o))
        self.kv_block, self.value_keys = most, _up(keys, RANGE)
        for width, block, enough in ((WIDE_RANGE, most, target), (WIDE_RANGE, 2, target), (RANGE, 2, target), (RANGE, 1, target // 2)):
            units = self.groups * -(-s.kv_heads // self.kv_block) * -(-keys // self.value_keys)
            if units >= enough:
                break
            self.kv_block = min(self.kv_block, block)
            units = self.groups * -(-s.kv_heads // self.kv_block)
            ranges = max(1, min(MOST_RANGES, -(-target // units), keys // width, room))
            self.value_keys = _up(-(-keys // ranges), RANGE)
        self.value_ranges = -(-keys // self.value_keys)
        rows = self.groups * tokens
        self.e_numel, self.sums_numel = rows * row_e, rows * inner * self.score_ranges
        self.partial_numel = rows * row_o * self.value_ranges


@register_part("mixer", "head_mix_attention")
class HeadMixAttention:
    graph_safe = True

    def __init__(self, spec):
        s = self.spec = spec
        if s.kv_heads < 1 or s.q_heads % s.kv_heads != 0:
            raise PartError(f"q_heads {s.q_heads} is no multiple of kv_heads {s.kv_heads}")
        if s.qk_norm is not None and s.qk_norm.size != s.head_dim:
            raise PartError("the q/k norm must span one head")
        if s.softcap is not None and not s.softcap > 0:
            raise PartError("the cap on the scores must be positive")
        if s.head_gate not in (None, "sigmoid"):
            raise PartError(f"head_gate {s.head_gate!r}: sigmoid or none")
        if s.value_position is not None and (s.value_position.dim != s.value_dim or s.value_dim % 2 != 0):
            raise PartError("turned values turn whole: an even value_dim with a position part as wide")
        if isinstance(s.sink, str) and s.sink != "learned":
            raise PartError(f"sink {s.sink!r}: a number, `learned` or none")
        self.position = build_part("position", s.position) if s.position is not None else None
        self.value_position = build_part("position", s.value_position) if s.value_position is not None else None
        self.q_width, self.k_width, self.v_width = s.q_heads * s.head_dim, s.kv_heads * s.head_dim, s.kv_heads * s.value_dim
        self.o_width = s.q_heads * s.value_dim
        self.out_name = "mixer_out"
        self.proj = self.o = self.q_norm = self.k_norm = self.sink = self.mix = None
        self._layouts = {}

    def _names(self):
        return ("q", "k", "v") + (("g",) if self.spec.head_gate is not None else ())

    def weight_specs(self):
        s = self.spec
        # (the gates ride behind q, k, v: one projection gives all four)
        specs = {"q": WeightSpec((self.q_width, s.hidden), stack="proj"), "k": WeightSpec((self.k_width, s.hidden), stack="proj"),
                 "v": WeightSpec((self.v_width, s.hidden), stack="proj")}
        if s.head_gate is not None:
            specs["g"] = WeightSpec((s.q_heads, s.hidden), stack="proj")
        specs["o"] = WeightSpec((s.hidden, self.o_width))
        specs["talk"] = WeightSpec((s.q_heads, s.q_heads), keep_float32=True, init=("normal", 0.0, float(s.q_heads) ** -0.5))
        if s.qk_norm is not None:
            specs["q.norm"] = WeightSpec((s.head_dim,), keep_float32=True)
            specs["k.norm"] = WeightSpec((s.head_dim,), keep_float32=True)
        if s.sink == "learned":
            specs["sink"] = WeightSpec((s.q_heads,), keep_float32=True, init=("normal", 0.0, 1.0))
        return specs

    def bind(self, weights):
        s = self.spec
        self.proj = stacked([weights[n] for n in self._names()])
        self.o, self.mix = weights["o"], weights["talk"]
        if s.qk_norm is not None:
            self.q_norm, self.k_norm = weights["q.norm"], weights["k.norm"]
        self.sink = weights["sink"] if s.sink == "learned" else s.sink

    def cache_spec(self):
        s = self.spec
        return PagedSpec((("k", (s.kv_heads, PAGE, s.head_dim)), ("v", (s.kv_heads, s.value_dim, PAGE))))

    def libraries(self):
        return ["gemm", "sink_attention", "head_mix_attention"]

    def check_limits(self, kernels, max_length, page_size, split_keys):
        s = self.spec
        if not kernels.head_mix_tiles_supported(s.q_heads, s.kv_heads, s.head_dim, s.value_dim, page_size, s.softcap) and \
                (130 * s.q_heads + self.o_width) * 4 > 150 * 1024:
            raise PartError(f"attention with mixed heads: {s.q_heads} heads of {s.value_dim} value channels are more than a "
                            "workgroup keeps")

    def _layout(self):
        s = self.spec
        if "it" not in self._layouts:
            from ..kernels.ops import Kernels
            self._layouts["it"] = Kernels.head_mix_layout(s.q_heads, s.kv_heads, s.value_dim)
        return self._layouts["it"]

    def workspace_plan(self, rows, dtype, limits):
        s = self.spec
        plan = {("mix_proj", dtype): rows * (self.q_width + self.k_width + self.v_width + (s.q_heads if s.head_gate else 0)),
                ("q", dtype): rows * self.q_width, ("attn", dtype): rows * self.o_width, (self.out_name, dtype): rows * s.hidden}
        layout = self._layout()
        if dtype == torch.bfloat16 and layout is not None and s.softcap is not None:
            inner = layout[1]
            keys = _up(int((limits or {}).get("max_length") or 1), 32)
            plan[(f"token_groups_1_{GROUP}", torch.int32)] = 2 * rows + 2
            # (a portion of two tokens takes a whole group of scratch rows)
            plan[("mix_e", dtype)] = max(GROUP * keys * inner, min(SCRATCH_CAP, rows * GROUP * keys * inner))
            plan[("mix_sums", torch.float32)] = min(SUMS_CAP, rows * GROUP * inner * MOST_RANGES)
            plan[("mix_partial", torch.float32)] = max(GROUP * self.o_width, min(PARTIAL_CAP, rows * GROUP * self.o_width * MOST_RANGES))
        return plan

    def forward(self, ctx, x, cache_id, write_cache=True):
        s = self.spec
        k = ctx.kernels
        m = x.shape[0]
        proj = ctx.workspace.get("mix_proj", (m, self.proj.shape[0]), x.dtype)
        k.gemm(x, self.proj, proj)
        view = ctx.cache.paged_view(cache_id)
        k_pages, v_pages = view.tensors["k"], view.tensors["v"]
        q = ctx.workspace.get("q", (m, self.q_width), x.dtype)
        rope, interleaved = _rope_table(self.position, ctx, x.device, s.head_dim)
        v_rope, v_interleaved = _rope_table(self.value_position, ctx, x.device, s.value_dim)
        k.sink_qkv_prep(proj, None, q, k_pages, v_pages, view.block_table, ctx.slots, ctx.positions, self.q_norm, self.k_norm,
                        s.qk_norm.eps if s.qk_norm is not None else 0.0, rope, s.q_heads, s.kv_heads, s.head_dim, s.value_dim,
                        view.page_size, write_cache, norm="before" if s.qk_norm is not None else None, interleaved=interleaved,
                        v_rope=v_rope, v_interleaved=v_interleaved, v_transposed=True)
        attn = ctx.workspace.get("attn", (m, self.o_width), x.dtype)
        gate = proj[:, self.q_width + self.k_width + self.v_width:] if s.head_gate is not None else None
        self._attend(ctx, q, k_pages, v_pages, view, (v_rope, v_interleaved) if v_rope is not None else None, gate, attn)
        out = ctx.workspace.get(self.out_name, (m, s.hidden), x.dtype)
        k.gemm(attn, self.o, out)
        return out

    def _attend(self, ctx, q, k_pages, v_pages, view, v_rope, gate, attn):
        s = self.spec
        k = ctx.kernels
        sizes = (s.q_heads, s.kv_heads, s.head_dim, s.value_dim, view.page_size)
        if not k.head_mix_tiles_supported(*sizes, s.softcap):
            k.head_mix_attention(q, k_pages, v_pages, view.block_table, ctx.slots, ctx.positions, self.mix, self.sink, v_rope,
                                 gate, attn, *sizes, float(s.scale), s.softcap)
            return
        small, big, _ = ctx.token_groups(1, GROUP)
        for (first, count, n), tokens in ((big, GROUP), (small, 1)):
            if n == 0:
                continue
            shape = LaunchShape(s, self._layout(), n, tokens, ctx.max_context, ctx.target_workgroups // 2)
            e = ctx.workspace.get("mix_e", (shape.e_numel,), q.dtype)
            sums = ctx.workspace.get("mix_sums", (shape.sums_numel,), torch.float32)
            partial = ctx.workspace.get("mix_partial", (shape.partial_numel,), torch.float32)
            for at in range(0, n, shape.groups):
                some = min(shape.groups, n - at)
                k.head_mix_tiles(q, k_pages, v_pages, view.block_table, ctx.slots, ctx.positions, self.mix, self.sink, v_rope,
                                 gate, attn, first[at:at + some], count[at:at + some], some, tokens, *sizes, float(s.scale),
                                 float(s.softcap), e, sums, partial, shape.ktiles, shape.score_keys, shape.score_ranges,
                                 shape.value_keys, shape.value_ranges, shape.kv_block)
