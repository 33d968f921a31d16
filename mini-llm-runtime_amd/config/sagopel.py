"""Sagopel: a pre-norm decoder whose sublayers join the stream with one factor, x <- x + m mixer(norm1(x));
x <- x + m ffn(norm2(x)).  A layer's mixer is one of
  `lightning`   linear attention with a constant decay a head on silu'd projections, the heads normed as one row and
                gated by a sigmoid;
  `parallel`    half the sum of two mixers' outputs, each normed over the model's width first: grouped-query attention
                over a sliding window that keeps the sequence's first tokens (biased q/k/v, a norm per head of q and k, a
                split-half rotation of a head's first channels, capped scores), and retention (the same recurrence on
                rotated q and k, each head over its own root mean square, gated by silu);
its feed-forward a gated one with relu, a mixture of gated silu experts (softmax scores, a choice corrected by a stored
number an expert, weights as they are, some choices standing for "the input as it is") beside a shared one, or none.
`loop` {start, stop, times} runs the layers start .. stop-1 `times` times in a row on the same tensors, every pass against
caches and states of its own, and adds a learned vector of its own to the stream before every pass (tensor `loop.step`).
The output is the final norm and the embedding table as the head.  This class knows the config.json keys and the tensor
names and nothing else: every size and constant goes through a spec to a registered part.

config.json: `architecture` (the name), `vocab`, `width`, `norm.eps`, `residual_mult`, optionally `loop`, and `layers`, a
list of {`type`, `mixer`: sizes and constants, `mlp`: null or {`kind`: dense, `ff`} or {`kind`: moe, `expert.ff`,
`router.experts`, `router.top`, `router.identity`, `shared.ff`}}.  Positions are not bounded by the model;
`max_positions`, when a file gives it, bounds what the engine plans for.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional, Tuple

from .pamunex import _object, _rotation
from .registry import ConfigError, register_architecture
from .specs import (DecayedLinearAttentionSpec, LayerRun, LayerSpec, MaskSpec, MixerSumSpec, MlpSpec, ModelSpec, NormSpec,
                    RoutedMlpSpec, RunVectorsSpec, SinkAttentionSpec)
from .taletar import DEFAULT_MAX_POSITIONS, _freeze, _int, _num, _thaw

HALF = 0.5                     # the share of either mixer in `parallel`


def _turned(m, where, dim):
    position = _rotation(m, where)
    if position.dim > dim:
        raise ConfigError(f"config.json: {where}rot.dims {position.dim} exceeds dim {dim}")
    return position


def _decays(m, heads, where):
    decay = m.get("decay")
    if not isinstance(decay, (list, tuple)) or len(decay) != heads or \
            not all(isinstance(d, (int, float)) and not isinstance(d, bool) and 0.0 < d <= 1.0 for d in decay):
        raise ConfigError(f"config.json: {where}decay must list one number in (0, 1] for each of the {heads} heads")
    return tuple(float(d) for d in decay)


def _lightning(m, width, eps, where):
    heads = _int(m, "heads", where)
    return DecayedLinearAttentionSpec(kind="decayed_linear_attention", hidden=width, heads=heads, head_dim=_int(m, "dim", where),
                                      value_dim=_int(m, "vdim", where), decay=_decays(m, heads, where), eps=eps,
                                      activation="silu", gate="sigmoid")


def _retention(m, width, eps, where):
    heads, dim = _int(m, "heads", where), _int(m, "dim", where)
    return DecayedLinearAttentionSpec(kind="decayed_linear_attention", hidden=width, heads=heads, head_dim=dim,
                                      value_dim=_int(m, "vdim", where), decay=_decays(m, heads, where), eps=eps,
                                      activation=None, gate="silu", position=_turned(m, where, dim), k_scale=float(dim) ** -0.5,
                                      norm="heads")


def _window_attention(m, width, eps, where):
    heads, kv = _int(m, "heads", where), _int(m, "kv_heads", where)
    if heads % kv != 0:
        raise ConfigError(f"config.json: {where}heads {heads} is no multiple of kv_heads {kv}")
    dim, mask = _int(m, "dim", where), _object(m, "mask", where)
    window = MaskSpec("window", _int(mask, "size", where + "mask."),
                      _int(mask, "keep_first", where + "mask.", lo=0) if "keep_first" in mask else 0)
    cap = None if m.get("softcap") is None else _num(m, "softcap", where, positive=True)
    return SinkAttentionSpec(kind="sink_attention", hidden=width, q_heads=heads, kv_heads=kv, head_dim=dim,
                             value_dim=_int(m, "vdim", where), scale=_num(m, "scale", where),
                             qk_norm=NormSpec("rmsnorm", dim, eps), position=_turned(m, where, dim), mask=window,
                             sink=False, bias=True, softcap=cap)


def _parallel(m, width, eps, where):
    left = _window_attention(_object(m, "left", where), width, eps, where + "left.")
    right = _retention(_object(m, "right", where), width, eps, where + "right.")
    return MixerSumSpec("mixer_sum", width, (("left", left, HALF), ("right", right, HALF)), out_norm_eps=eps)


def _mlp(mlp, width, where):
    if mlp is None:
        return None
    if not isinstance(mlp, dict) or mlp.get("kind") not in ("dense", "moe"):
        raise ConfigError(f"config.json: {where} must be null or an object of kind `dense` or `moe`")
    if mlp["kind"] == "dense":
        return MlpSpec("swiglu", width, _int(mlp, "ff", where + "."), "relu")
    expert, router = _object(mlp, "expert", where + "."), _object(mlp, "router", where + ".")
    at = where + ".router."
    experts, top = _int(router, "experts", at), _int(router, "top", at)
    identity = _int(router, "identity", at, lo=0) if "identity" in router else 0
    if top > experts + identity:
        raise ConfigError(f"config.json: {where}.router: {top} choices among {experts} experts and {identity} identities")
    shared = None
    if mlp.get("shared") is not None:
        shared = MlpSpec("swiglu", width, _int(_object(mlp, "shared", where + "."), "ff", where + ".shared."), "silu")
    return RoutedMlpSpec("routed_mlp", width, _int(expert, "ff", where + ".expert."), experts, top, 1, 1, "silu", "softmax",
                         False, gated=True, correction=True, shared=shared, identity=identity)


_MIXERS = {"lightning": _lightning, "parallel": _parallel}
_FFN_TENSORS = {"gate_proj": "gate", "up_proj": "up", "down_proj": "down"}


@register_architecture("Sagopel")
@dataclass(frozen=True)
class SagopelConfig:
    vocab: int
    width: int
    eps: float
    residual_mult: float
    layers: Tuple                        # the `layers` list of config.json, frozen
    loop: Optional[Tuple[int, int, int]] = None     # (start, stop, times)
    max_positions: int = DEFAULT_MAX_POSITIONS
    eos_token_ids: Tuple[int, ...] = ()

    @classmethod
    def from_dict(cls, data):
        for key in ("vocab", "width", "norm", "layers"):
            if key not in data:
                raise ConfigError(f"config.json: missing `{key}`")
        if not isinstance(data["norm"], dict):
            raise ConfigError("config.json: `norm` must be an object with `eps`")
        layers = data["layers"]
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: `layers` must be a non-empty list")
        width = _int(data, "width", "")
        for i, layer in enumerate(layers):
            where = f"layers[{i}]."
            if not isinstance(layer, dict) or not isinstance(layer.get("mixer"), dict):
                raise ConfigError(f"config.json: {where}mixer must be an object")
            if layer.get("type") not in _MIXERS:
                raise ConfigError(f"config.json: {where}type {layer.get('type')!r} is none of {sorted(_MIXERS)}")
            _MIXERS[layer["type"]](layer["mixer"], width, 1e-6, where + "mixer.")      # (checks the keys)
            _mlp(layer.get("mlp"), width, where + "mlp")
        loop = None
        if data.get("loop") is not None:
            lp = _object(data, "loop", "")
            loop = (_int(lp, "start", "loop.", lo=0, hi=len(layers)), _int(lp, "stop", "loop.", lo=0, hi=len(layers)),
                    _int(lp, "times", "loop.", lo=1))
            if loop[0] > loop[1]:
                raise ConfigError(f"config.json: loop.start {loop[0]} lies behind loop.stop {loop[1]}")
        eos = data.get("eos_token_id")
        eos_ids = () if eos is None else (eos,) if isinstance(eos, int) else tuple(eos)
        return cls(vocab=_int(data, "vocab", ""), width=width, eps=_num(data["norm"], "eps", "norm.", positive=True),
                   residual_mult=_num(data, "residual_mult", "", default=1.0), layers=_freeze(layers), loop=loop,
                   max_positions=_int(data, "max_positions", "") if "max_positions" in data else DEFAULT_MAX_POSITIONS,
                   eos_token_ids=eos_ids)

    def to_dict(self):
        out = {"architecture": self.architecture, "layers": _thaw(self.layers), "norm": {"eps": self.eps},
               "residual_mult": self.residual_mult, "vocab": self.vocab, "width": self.width}
        if self.loop is not None:
            out["loop"] = {"start": self.loop[0], "stop": self.loop[1], "times": self.loop[2]}
        if self.max_positions != DEFAULT_MAX_POSITIONS:
            out["max_positions"] = self.max_positions
        if self.eos_token_ids:
            out["eos_token_id"] = list(self.eos_token_ids)
        return out

    # ---- the model as parts -------------------------------------------------------------------
    def run_order(self):
        """[(layer, the number of the pass that starts with this run, or None)] in the order the layers run."""
        start, stop, times = self.loop if self.loop is not None else (0, 0, 0)
        order = [(i, None) for i in range(start)]
        for p in range(times):
            order += [(i, p if i == start else None) for i in range(start, stop)]
        return order + [(i, None) for i in range(stop, len(self.layers))]

    def model_spec(self):
        norm = NormSpec("rmsnorm", self.width, self.eps)
        specs = []
        for i, layer in enumerate(_thaw(self.layers)):
            mixer = _MIXERS[layer["type"]](layer["mixer"], self.width, self.eps, f"layers[{i}].mixer.")
            ffn = _mlp(layer.get("mlp"), self.width, f"layers[{i}].mlp")
            specs.append(LayerSpec("prenorm", norm, mixer, None if ffn is None else norm, ffn, residual_scale=self.residual_mult))
        # every run has a cache entry of its own: a looped layer keeps what each of its passes saw
        schedule = tuple(LayerRun(layer, run, add_vector=step) for run, (layer, step) in enumerate(self.run_order()))
        vectors = RunVectorsSpec("run_vectors", self.loop[2], self.width) if self.loop is not None else None
        return ModelSpec(architecture=self.architecture, vocab_size=self.vocab, hidden=self.width, layers=tuple(specs),
                         schedule=schedule, final_norm=norm, tie_embeddings=True, max_positions=self.max_positions,
                         eos_token_ids=self.eos_token_ids, run_vectors=vectors)

    # ---- tensor names ----------------------------------------------------------------------------
    @staticmethod
    def global_tensor_name(local):
        return {"embed.weight": "embed", "final_norm.weight": "final.norm", "head.weight": "head",
                "run_vectors.weight": "loop.step"}[local]

    @staticmethod
    def layer_tensor_name(layer, part, local):
        if part in ("norm1", "norm2"):
            return f"l{layer}.{part}"
        if part == "mixer":
            return f"l{layer}.mix.{local}"
        head, dot, last = local.rpartition(".")
        return f"l{layer}.mlp.{head}{dot}{_FFN_TENSORS.get(last, last)}"
