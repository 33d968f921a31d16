"""A plain, slow implementation of the Nuvorax decoder in float64 numpy: whole sequences, no cache, no
batching, one function per mechanism.  It shares no code with the engine; the engine's tests compare
against it.

Notation: x [T, E] is the residual stream of one sequence, positions count from 0, linear weights are
[out, in] and applied as x @ W.T.  `cfg` is a mixer's (or feed-forward's) entry of config.json, `w` maps
the last part of a tensor's name ("q", "talk", "e3.up", "shared.sg", ...) to an array.
"""
from __future__ import annotations

import math

import numpy as np

SLOPE = 1.702        # of the experts' gate


def layer_norm(x, weight, eps):
    mu = x.mean(axis=-1, keepdims=True)
    spread = ((x - mu) ** 2).mean(axis=-1, keepdims=True)
    return (x - mu) / np.sqrt(spread + eps) * weight


def rms_norm(x, weight, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * weight


def turn(x, angles):
    """x [T, heads, 2 n]: channel i paired with channel i + n, the pair turned by angles[t, i]."""
    n = x.shape[-1] // 2
    c, s = np.cos(angles)[:, None, :], np.sin(angles)[:, None, :]
    u, v = x[..., :n], x[..., n:]
    return np.concatenate([u * c - v * s, v * c + u * s], axis=-1)


def plain_frequencies(dims, base):
    return base ** (-2.0 * np.arange(dims // 2) / dims)


def banded_frequencies(freq, scaling):
    """Every frequency by its wavelength 2 pi / f: short ones keep f, long ones get f / factor, and in between the
    two are blended by where original / wavelength lies between `low` and `high`."""
    out = []
    for f in freq:
        turns = scaling["original"] * f / (2.0 * math.pi)            # original length over the wavelength
        if turns > scaling["high"]:
            out.append(f)
        elif turns < scaling["low"]:
            out.append(f / scaling["factor"])
        else:
            s = (turns - scaling["low"]) / (scaling["high"] - scaling["low"])
            out.append((1.0 - s) * f / scaling["factor"] + s * f)
    return np.array(out)


def rotate_keys(x, positions, rot):
    """The first `dims` channels of every head turned; the others pass."""
    freq = plain_frequencies(rot["dims"], rot["base"])
    if rot.get("scaling") is not None:
        freq = banded_frequencies(freq, rot["scaling"])
    angles = np.asarray(positions, dtype=np.float64)[:, None] * freq[None, :]
    return np.concatenate([turn(x[..., :rot["dims"]], angles), x[..., rot["dims"]:]], axis=-1)


def rotate_values(v, positions, base, direction=1.0):
    """All channels of a value (or, with direction -1, of an output) turned by its position, never stretched."""
    freq = plain_frequencies(v.shape[-1], base)
    return turn(v, direction * np.asarray(positions, dtype=np.float64)[:, None] * freq[None, :])


def capped(scores, cap):
    return cap * np.tanh(scores / cap)


def softmax_plus_one(scores, seen):
    """exp(s) over one plus their sum: as if one more key scored 0 and brought nothing."""
    s = np.where(seen, scores, -np.inf)
    top = np.maximum(s.max(axis=-1, keepdims=True), 0.0)
    e = np.exp(s - top)
    return e / (np.exp(-top) + e.sum(axis=-1, keepdims=True))


def mixed_heads(weights, talk):
    """weights [H, T, T]: head h's becomes sum_g talk[h, g] weights[g]."""
    return np.tensordot(talk, weights, axes=([1], [0]))


def attention_heads(q, k, v, positions, cfg, talk):
    """The mixer between its projections and its gate: q, k normed and turned, v turned -> [T, H, V], turned back."""
    H, G = cfg["heads"], cfg["kv_heads"]
    seen = np.tril(np.ones((q.shape[0], q.shape[0]), dtype=bool))
    weights = np.stack([softmax_plus_one(capped((q[:, h] @ k[:, h // (H // G)].T) * cfg["scale"], cfg["softcap"]), seen)
                        for h in range(H)])
    weights = mixed_heads(weights, talk)
    out = np.stack([weights[h] @ v[:, h // (H // G)] for h in range(H)], axis=1)
    return rotate_values(out, positions, cfg["rot"]["base"], -1.0)


def attention(x, w, cfg, eps, positions=None):
    T = x.shape[0]
    positions = np.arange(T) if positions is None else positions
    H, G, D, V = cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    q = rms_norm((x @ w["q"].T).reshape(T, H, D), w["q.norm"], eps)
    k = rms_norm((x @ w["k"].T).reshape(T, G, D), w["k.norm"], eps)
    v = (x @ w["v"].T).reshape(T, G, V)
    q, k = rotate_keys(q, positions, cfg["rot"]), rotate_keys(k, positions, cfg["rot"])
    v = rotate_values(v, positions, cfg["rot"]["base"])
    out = attention_heads(q, k, v, positions, cfg, w["talk"])
    gate = 1.0 / (1.0 + np.exp(-(x @ w["g"].T)))
    return (out * gate[:, :, None]).reshape(T, H * V) @ w["o"].T


def gelu_erf(z):
    return 0.5 * z * (1.0 + np.vectorize(math.erf, otypes=[float])(z / math.sqrt(2.0)))


def dense_ffn(x, w):
    return gelu_erf(x @ w["up"].T) @ w["down"].T


def clamped_glu(x, gate, up, down, limit):
    g = np.minimum(x @ gate.T, limit)
    u = np.clip(x @ up.T, -limit, limit)
    return (g / (1.0 + np.exp(-SLOPE * g)) * (u + 1.0)) @ down.T


def softmax(z):
    e = np.exp(z - z.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def route(x, w, router):
    """(chosen experts [T, top], their weights [T, top])."""
    n, top = router["experts"], router["top"]
    groups = router.get("groups") or {"count": 1, "keep": 1}
    per = n // groups["count"]
    s = softmax(x @ w["router"].T)
    chosen, weights = [], []
    for row in s:
        best = [row[g * per:(g + 1) * per].max() for g in range(groups["count"])]
        kept = sorted(range(groups["count"]), key=lambda g: (-best[g], g))[:groups["keep"]]
        allowed = [e for e in range(n) if e // per in kept]
        picks = sorted(allowed, key=lambda e: (-row[e], e))[:top]
        chosen.append(picks)
        weights.append(row[picks] / (row[picks].sum() + 1e-20) * router["scale"])
    return np.array(chosen), np.array(weights)


def route_margin(x, w, router, rounding=2.0 ** -8):
    """[T]: how far each token's choice is from another one, in units of what rounding x (relative, per element) may
    move a router logit: the gap between the last group kept and the first one dropped, and between the last expert
    chosen and the best one left (infinite where nothing is left out).  (A softmax keeps the logits' order.)"""
    n, top = router["experts"], router["top"]
    groups = router.get("groups") or {"count": 1, "keep": 1}
    per, keep = n // groups["count"], groups["keep"]
    z = x @ w["router"].T
    moved = (rounding * np.sqrt((x * x) @ (w["router"] ** 2).T)).max(axis=1) + 1e-300
    gaps = []
    for row in z:
        best = [row[g * per:(g + 1) * per].max() for g in range(groups["count"])]
        order = sorted(range(groups["count"]), key=lambda g: (-best[g], g))
        gap = best[order[keep - 1]] - best[order[keep]] if keep < groups["count"] else np.inf
        ranked = sorted((row[e] for e in range(n) if e // per in order[:keep]), reverse=True)
        if top < len(ranked):
            gap = min(gap, ranked[top - 1] - ranked[top])
        gaps.append(gap)
    return np.array(gaps) / moved


def moe_ffn(x, w, cfg):
    chosen, weights = route(x, w, cfg["router"])
    out = np.zeros_like(x)
    for e in range(cfg["router"]["experts"]):
        rows, place = np.nonzero(chosen == e)
        if len(rows):
            y = clamped_glu(x[rows], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"], cfg["expert"]["limit"])
            out[rows] += weights[rows, place][:, None] * y
    if cfg.get("shared") is not None:
        y = clamped_glu(x, w["shared.gate"], w["shared.up"], w["shared.down"], cfg["shared"]["limit"])
        out = out + y / (1.0 + np.exp(-(x @ w["shared.sg"].T)))
    return out


def feed_forward(x, w, cfg):
    return dense_ffn(x, w) if cfg["kind"] == "dense" else moe_ffn(x, w, cfg)


def layer_weights(weights, layer, part):
    prefix = f"l{layer}.{part}."
    return {name[len(prefix):]: value for name, value in weights.items() if name.startswith(prefix)}


def forward(config, weights, tokens, streams=None, margins=None):
    """Logits [T, vocab] of one sequence from position 0.  `weights`: {tensor name: float64 array}.
    `streams`, a list, receives the residual stream after every layer; `margins`, a list, the routing margin
    [T] of every layer that routes."""
    eps = config["norm"]["eps"]
    x = weights["embed"][np.asarray(tokens)] * config["embedding"]["scale"]
    for i, layer in enumerate(config["layers"]):
        h = layer_norm(x, weights[f"l{i}.norm1"], eps)
        delta = attention(h, layer_weights(weights, i, "mix"), layer["mixer"], eps)
        mlp = layer.get("mlp")
        if mlp is not None:
            w = layer_weights(weights, i, "mlp")
            delta = delta + feed_forward(h, w, mlp)
            if margins is not None and mlp["kind"] == "moe":
                margins.append(route_margin(h, w, mlp["router"]))
        x = x + delta
        if streams is not None:
            streams.append(x.copy())
    return (layer_norm(x, weights["final.norm"], eps) @ weights["head"].T) * config["logit_scale"]


class PlainNuvorax:
    """A model folder (config.json, model.safetensors) run by the functions above."""

    def __init__(self, folder):
        import json
        import os

        import torch
        from safetensors.torch import load_file
        with open(os.path.join(folder, "config.json")) as f:
            self.cfg = json.load(f)
        self.tensors = {n: (t.to(torch.float64) if t.dtype.is_floating_point else t).numpy()
                        for n, t in load_file(os.path.join(folder, "model.safetensors")).items()}

    def logits(self, tokens, want=None):
        rows = forward(self.cfg, self.tensors, tokens)
        return rows if want is None else rows[np.asarray(want, dtype=np.int64)]

    def streams(self, tokens):
        out = []
        forward(self.cfg, self.tensors, tokens, streams=out)
        return np.stack(out)

    def routing_margins(self, tokens):
        """[T]: the smallest routing margin of every position over the layers that route (see `route_margin`);
        None for a model that routes nowhere."""
        margins = []
        forward(self.cfg, self.tensors, tokens, margins=margins)
        return np.min(margins, axis=0) if margins else None

    def decisive(self, tokens, rng, least=40.0, tries=400):
        """`tokens` with every position whose routing is a close call (a margin below `least`) drawn again, until
        none is left: no comparison with an engine that rounds then rests on a close call.  (A position's margins
        depend on the tokens up to it only, so what lies before the first close call stays as it is; the others are
        drawn again in the same pass, which usually settles many at once.)"""
        tokens = list(tokens)
        vocab = self.tensors["embed"].shape[0]
        for _ in range(tries):
            margins = self.routing_margins(tokens)
            near = [] if margins is None else np.nonzero(margins < least)[0]
            if len(near) == 0:
                return tokens
            for t in near:
                tokens[int(t)] = int(rng.integers(0, vocab))
        raise ValueError("no decisive sequence found")

    def greedy(self, prompt, n):
        tokens, out = list(prompt), []
        for _ in range(n):
            t = int(np.argmax(self.logits(tokens, [len(tokens) - 1])[0]))
            out.append(t)
            tokens.append(t)
        return out
