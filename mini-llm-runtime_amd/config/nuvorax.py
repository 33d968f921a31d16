"""Nuvorax: a decoder whose sublayers stand side by side behind ONE layer norm without a bias, x <- x + (mixer(h) + ffn(h))
with h = norm1(x).  The mixer is causal grouped-query attention with a norm per head of q and k, a rotation of a head's
first channels whose frequencies are scaled by bands, values turned by their position (a head's output is turned back),
capped scores, a softmax with one added to its denominator, softmax weights that are mixed between the heads before they
meet the values, and one sigmoid gate a head.  The feed-forward is an ungated gelu one, a mixture of clamped gated
experts (softmax scores, the best groups of neighbouring experts, the chosen scores over their sum times a factor)
beside a gated shared expert, or none.  The embedding has a factor, and so have the logits of an untied head.  This
class knows the config.json keys and the tensor names and nothing else: every size and constant goes through a spec to
a registered part.

config.json: `architecture` (the name), `vocab`, `width`, `norm.eps`, `embedding.scale`, `logit_scale`, and `layers`, a
list of {`type`: attention, `mixer`: sizes and constants (`heads`, `kv_heads`, `dim`, `vdim`, `scale`, `softcap`,
`rot.base`, `rot.dims`, `rot.scaling` {`factor`, `low`, `high`, `original`}), `mlp`: null, {`kind`: dense, `ff`} or
{`kind`: moe, `expert` {`ff`, `limit`}, `router` {`experts`, `top`, `groups` {`count`, `keep`}, `scale`}, `shared` {`ff`,
`limit`}}}.  Positions are not bounded by the model; `max_positions`, when a file gives it, bounds what the engine plans
for.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Tuple

from .pamunex import _object
from .registry import ConfigError, register_architecture
from .specs import (ClampedGluSpec, EmbedSpec, FrequencyBands, HeadMixAttentionSpec, HeadSpec, LayerRun, LayerSpec, ModelSpec,
                    NormSpec, PlainMlpSpec, PositionSpec, RoutedMlpSpec)
from .taletar import DEFAULT_MAX_POSITIONS, _freeze, _int, _num, _thaw

SINK = 0.0                     # the score of the softmax's valueless summand: one is added to the denominator
GATE_SLOPE = 1.702             # of the experts' clamped gate


def _positions(m, dim, vdim, where):
    """(the rotation of q and k, the rotation of the values: all channels, the same base, never scaled)."""
    rot = _object(m, "rot", where)
    dims = _int(rot, "dims", where + "rot.")
    if dims % 2 != 0 or dims > dim:
        raise ConfigError(f"config.json: {where}rot.dims {dims} must be even and at most dim {dim}")
    if vdim % 2 != 0:
        raise ConfigError(f"config.json: {where}vdim {vdim} must be even: values are turned in pairs")
    base = _num(rot, "base", where + "rot.", positive=True)
    bands = None
    if rot.get("scaling") is not None:
        sc, at = _object(rot, "scaling", where + "rot."), where + "rot.scaling."
        bands = FrequencyBands(factor=_num(sc, "factor", at, positive=True), original=_num(sc, "original", at, positive=True),
                               low=_num(sc, "low", at, positive=True), high=_num(sc, "high", at, positive=True))
        if bands.high < bands.low:
            raise ConfigError(f"config.json: {at}high {bands.high} lies below low {bands.low}")
    return PositionSpec("rope", dims, base, bands=bands), PositionSpec("rope", vdim, base)


def _attention(m, width, eps, where):
    heads, kv = _int(m, "heads", where), _int(m, "kv_heads", where)
    if heads % kv != 0:
        raise ConfigError(f"config.json: {where}heads {heads} is no multiple of kv_heads {kv}")
    dim, vdim = _int(m, "dim", where), _int(m, "vdim", where)
    position, value_position = _positions(m, dim, vdim, where)
    softcap = None if m.get("softcap") is None else _num(m, "softcap", where, positive=True)
    return HeadMixAttentionSpec(kind="head_mix_attention", hidden=width, q_heads=heads, kv_heads=kv, head_dim=dim,
                                value_dim=vdim, scale=_num(m, "scale", where), softcap=softcap,
                                qk_norm=NormSpec("rmsnorm", dim, eps), position=position, value_position=value_position,
                                sink=SINK, head_gate="sigmoid")


def _mlp(mlp, width, where):
    if mlp is None:
        return None
    if not isinstance(mlp, dict) or mlp.get("kind") not in ("dense", "moe"):
        raise ConfigError(f"config.json: {where} must be null or an object of kind `dense` or `moe`")
    if mlp["kind"] == "dense":
        return PlainMlpSpec("plain_mlp", width, _int(mlp, "ff", where + "."), "gelu_erf")
    expert, router = _object(mlp, "expert", where + "."), _object(mlp, "router", where + ".")
    groups = router.get("groups") or {"count": 1, "keep": 1}
    experts, top = _int(router, "experts", where + ".router."), _int(router, "top", where + ".router.")
    count, keep = _int(groups, "count", where + ".router.groups."), _int(groups, "keep", where + ".router.groups.")
    if experts % count != 0 or keep > count or top > keep * (experts // count):
        raise ConfigError(f"config.json: {where}.router: {experts} experts in {count} groups of which {keep} stay "
                          f"cannot give {top} choices")
    shared = None
    if mlp.get("shared") is not None:
        sh = _object(mlp, "shared", where + ".")
        shared = ClampedGluSpec("clamped_glu", width, _int(sh, "ff", where + ".shared."),
                                _num(sh, "limit", where + ".shared.", positive=True), GATE_SLOPE)
    return RoutedMlpSpec("routed_mlp", width, _int(expert, "ff", where + ".expert."), experts, top, count, keep, "clamped",
                         "softmax", True, gated=True, group_score="best", limit=_num(expert, "limit", where + ".expert.", positive=True),
                         slope=GATE_SLOPE, route_scale=_num(router, "scale", where + ".router.", default=1.0), shared=shared,
                         shared_gate=shared is not None)


_MIXERS = {"attention": _attention}


@register_architecture("Nuvorax")
@dataclass(frozen=True)
class NuvoraxConfig:
    vocab: int
    width: int
    eps: float
    layers: Tuple                        # the `layers` list of config.json, frozen
    embedding_scale: float = 1.0
    logit_scale: float = 1.0
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
        embedding = _object(data, "embedding", "") if data.get("embedding") is not None else {}
        eos = data.get("eos_token_id")
        eos_ids = () if eos is None else (eos,) if isinstance(eos, int) else tuple(eos)
        return cls(vocab=_int(data, "vocab", ""), width=width, eps=_num(data["norm"], "eps", "norm.", positive=True),
                   layers=_freeze(layers), embedding_scale=_num(embedding, "scale", "embedding.", default=1.0),
                   logit_scale=_num(data, "logit_scale", "", default=1.0),
                   max_positions=_int(data, "max_positions", "") if "max_positions" in data else DEFAULT_MAX_POSITIONS,
                   eos_token_ids=eos_ids)

    def to_dict(self):
        out = {"architecture": self.architecture, "embedding": {"scale": self.embedding_scale}, "layers": _thaw(self.layers),
               "logit_scale": self.logit_scale, "norm": {"eps": self.eps}, "vocab": self.vocab, "width": self.width}
        if self.max_positions != DEFAULT_MAX_POSITIONS:
            out["max_positions"] = self.max_positions
        if self.eos_token_ids:
            out["eos_token_id"] = list(self.eos_token_ids)
        return out

    # ---- the model as parts -------------------------------------------------------------------
    def model_spec(self):
        norm = NormSpec("layernorm", self.width, self.eps, bias=False)
        specs = []
        for i, layer in enumerate(_thaw(self.layers)):
            mixer = _MIXERS[layer["type"]](layer["mixer"], self.width, self.eps, f"layers[{i}].mixer.")
            specs.append(LayerSpec("parallel", norm, mixer, None, _mlp(layer.get("mlp"), self.width, f"layers[{i}].mlp")))
        return ModelSpec(architecture=self.architecture, vocab_size=self.vocab, hidden=self.width, layers=tuple(specs),
                         schedule=tuple(LayerRun(i, i) for i in range(len(specs))), final_norm=norm, tie_embeddings=False,
                         max_positions=self.max_positions, eos_token_ids=self.eos_token_ids,
                         embed=EmbedSpec("token_embedding", self.vocab, self.width, scale=self.embedding_scale),
                         head=HeadSpec("scaled_head", self.vocab, self.width, tied=False, scale=self.logit_scale))

    # ---- tensor names ----------------------------------------------------------------------------
    @staticmethod
    def global_tensor_name(local):
        return {"embed.weight": "embed", "final_norm.weight": "final.norm", "head.weight": "head"}[local]

    @staticmethod
    def layer_tensor_name(layer, part, local):
        if part == "norm1":
            return f"l{layer}.norm1"
        return f"l{layer}.{'mix' if part == 'mixer' else 'mlp'}.{local}"
