"""A plain, slow implementation of the Sagopel decoder in float64 numpy: whole sequences, no cache, no
batching, one function per mechanism.  It shares no code with the engine; the engine's tests compare
against it.

Notation: x [T, E] is the residual stream of one sequence, positions count from 0, linear weights are
[out, in] and applied as x @ W.T.  `cfg` is a mixer's (or feed-forward's) entry of config.json, `w` maps
the last part of a tensor's name ("q", "left.q.b", "router", "e3.up", ...) to an array.
"""
from __future__ import annotations

import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def relu(z):
    return np.maximum(z, 0.0)


def over_rms(x, eps):
    """Divided by the root of (the mean square along the last axis plus eps)."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def rms_norm(x, weight, eps):
    return over_rms(x, eps) * weight


def sub(w, prefix):
    """The tensors under a dotted prefix, by the rest of their names."""
    return {name[len(prefix) + 1:]: value for name, value in w.items() if name.startswith(prefix + ".")}


# ---- rotation ---------------------------------------------------------------------------------------------
def rotate(x, positions, dims, base):
    """x [T, heads, D]: the first `dims` channels of every head turned by the token's position in pairs
    (i, i + dims / 2); the other channels pass."""
    half = dims // 2
    f = base ** (-2.0 * np.arange(half, dtype=np.float64) / dims)
    angle = np.asarray(positions, dtype=np.float64)[:, None] * f[None, :]
    c, s = np.cos(angle)[:, None, :], np.sin(angle)[:, None, :]
    out = np.array(x, dtype=np.float64, copy=True)
    u, v = x[..., :half], x[..., half:dims]
    out[..., :half] = u * c - v * s
    out[..., half:dims] = v * c + u * s
    return out


# ---- softmax attention ------------------------------------------------------------------------------------
def seen_in_window(queries, keys, size, keep_first):
    """[queries, keys]: no key behind the query; the last `size` positions, and the first `keep_first` of the
    sequence."""
    p, j = np.asarray(queries)[:, None], np.asarray(keys)[None, :]
    return (j <= p) & ((p - j < size) | (j < keep_first))


def capped(scores, cap):
    return cap * np.tanh(scores / cap)


def masked_softmax(scores, seen):
    s = np.where(seen, scores, -np.inf)
    p = np.exp(s - s.max(axis=1, keepdims=True))
    return p / p.sum(axis=1, keepdims=True)


def attend(q, k, v, scale, cap, seen):
    """q [M, H, D] over keys k [T, G, D] and values v [T, G, V] -> [M, H * V]; query head h reads key/value head
    h // (H / G)."""
    H, G = q.shape[1], k.shape[1]
    heads = []
    for head in range(H):
        g = head // (H // G)
        heads.append(masked_softmax(capped((q[:, head] @ k[:, g].T) * scale, cap), seen) @ v[:, g])
    return np.concatenate(heads, axis=1)


def window_attention(x, w, cfg, eps):
    """Grouped-query attention over a sliding window and the sequence's first tokens: biased q/k/v, a norm per head of
    q and k, a rotation of a head's first channels, capped scores."""
    T = x.shape[0]
    H, G, D, V = cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    q = rms_norm((x @ w["q"].T + w["q.b"]).reshape(T, H, D), w["q.norm"], eps)
    k = rms_norm((x @ w["k"].T + w["k.b"]).reshape(T, G, D), w["k.norm"], eps)
    v = (x @ w["v"].T + w["v.b"]).reshape(T, G, V)
    pos = np.arange(T)
    q = rotate(q, pos, cfg["rot"]["dims"], cfg["rot"]["base"])
    k = rotate(k, pos, cfg["rot"]["dims"], cfg["rot"]["base"])
    seen = seen_in_window(pos, pos, cfg["mask"]["size"], cfg["mask"]["keep_first"])
    return attend(q, k, v, cfg["scale"], cfg["softcap"], seen) @ w["o"].T


# ---- recurrences ------------------------------------------------------------------------------------------
def decayed_sum(q, k, v, decay):
    """One head.  q, k [T, D], v [T, V]: S <- decay S + k v^T, o = S^T q, S = 0 at the start."""
    T, D = q.shape
    S = np.zeros((D, v.shape[1]))
    out = np.zeros((T, v.shape[1]))
    for t in range(T):
        S = decay * S + np.outer(k[t], v[t])
        out[t] = S.T @ q[t]
    return out


def lightning(x, w, cfg, eps):
    """Linear attention with a constant decay a head on silu'd projections; the heads side by side normed as one row,
    gated by a sigmoid, projected."""
    T = x.shape[0]
    H, D, V = cfg["heads"], cfg["dim"], cfg["vdim"]
    q, k = silu(x @ w["q"].T).reshape(T, H, D), silu(x @ w["k"].T).reshape(T, H, D)
    v = silu(x @ w["v"].T).reshape(T, H, V)
    o = np.concatenate([decayed_sum(q[:, h], k[:, h], v[:, h], cfg["decay"][h]) for h in range(H)], axis=1)
    return (rms_norm(o, w["norm"], eps) * sigmoid(x @ w["g"].T)) @ w["o"].T


def retention(x, w, cfg, eps):
    """The same recurrence on rotated q and k (k over the root of its size), each head's output over its root mean
    square, gated by silu, projected."""
    T = x.shape[0]
    H, D, V = cfg["heads"], cfg["dim"], cfg["vdim"]
    pos = np.arange(T)
    q = rotate((x @ w["q"].T).reshape(T, H, D), pos, cfg["rot"]["dims"], cfg["rot"]["base"])
    k = rotate((x @ w["k"].T).reshape(T, H, D), pos, cfg["rot"]["dims"], cfg["rot"]["base"]) * D ** -0.5
    v = (x @ w["v"].T).reshape(T, H, V)
    o = np.concatenate([over_rms(decayed_sum(q[:, h], k[:, h], v[:, h], cfg["decay"][h]), eps) for h in range(H)], axis=1)
    return (o * silu(x @ w["g"].T)) @ w["o"].T


def retention_margin(x, w, cfg, rounding=2.0 ** -9):
    """[T]: the smallest of a token's heads' outputs (root mean square), in units of what rounding q, k and v (relative, per
    element) may move it by: a head whose output nearly cancels is brought to size one all the same."""
    T = x.shape[0]
    H, D, V = cfg["heads"], cfg["dim"], cfg["vdim"]
    pos = np.arange(T)
    q, k = (rotate((x @ w[n].T).reshape(T, H, D), pos, cfg["rot"]["dims"], cfg["rot"]["base"]) for n in "qk")
    v = (x @ w["v"].T).reshape(T, H, V)
    size = lambda a: np.sqrt(np.mean(a * a, axis=1))
    return np.min([size(decayed_sum(q[:, h], k[:, h], v[:, h], cfg["decay"][h]))
                   / (rounding * size(decayed_sum(abs(q[:, h]), abs(k[:, h]), abs(v[:, h]), cfg["decay"][h]))) for h in range(H)], axis=0)


def two_mixers(x, w, cfg, eps):
    """Half the sum of two mixers' outputs, each normed over the model's width first."""
    left = window_attention(x, sub(w, "left"), cfg["left"], eps)
    right = retention(x, sub(w, "right"), cfg["right"], eps)
    return 0.5 * (rms_norm(left, w["left.out"], eps) + rms_norm(right, w["right.out"], eps))


# ---- feed-forwards ----------------------------------------------------------------------------------------
def gated_ffn(x, w, act):
    return (act(x @ w["gate"].T) * (x @ w["up"].T)) @ w["down"].T


def softmax_rows(z):
    e = np.exp(z - z.max(axis=1, keepdims=True))
    return e / e.sum(axis=1, keepdims=True)


def route(x, w, router):
    """(ids [T, top], weights [T, top]): the largest scores plus correction (ties: the lower number), weighted by the
    scores themselves."""
    s = softmax_rows(x @ w["router"].T)
    order = np.argsort(-(s + w["correction"]), axis=1, kind="stable")[:, :router["top"]]
    return order, np.take_along_axis(s, order, axis=1)


def route_margin(x, w, cfg, rounding=2.0 ** -8):
    """[T]: how far each token's choice is from another one, in units of what rounding x (relative, per element) may move
    a choice score: the gap between the last output chosen and the best one left (infinite where every one is chosen)."""
    top = cfg["router"]["top"]
    z = x @ w["router"].T
    if top >= z.shape[1]:
        return np.full(x.shape[0], np.inf)
    s = softmax_rows(z)
    c = s + w["correction"]
    moved = (rounding * np.sqrt((x * x) @ (w["router"] ** 2).T)).max(axis=1) + 1e-300
    order = np.argsort(-c, axis=1, kind="stable")
    at = lambda a, i: np.take_along_axis(a, order[:, i:i + 1], axis=1)[:, 0]
    return (at(c, top - 1) - at(c, top)) / (moved * (at(s, top - 1) + at(s, top)) + 1e-300)


def moe_ffn(x, w, cfg):
    """The chosen experts' weighted sum, the router's last `identity` outputs standing for experts that give their input
    back, plus the shared expert."""
    router = cfg["router"]
    ids, weights = route(x, w, router)
    out = gated_ffn(x, sub(w, "shared"), silu) if cfg.get("shared") is not None else np.zeros_like(x)
    for t in range(x.shape[0]):
        for e, g in zip(ids[t], weights[t]):
            out[t] = out[t] + g * (x[t] if e >= router["experts"] else gated_ffn(x[t:t + 1], sub(w, f"e{e}"), silu)[0])
    return out


MIXERS = {"lightning": lightning, "parallel": two_mixers}


def run_order(config):
    """[(layer, the pass's number when the run is a pass's first, else None)] in the order the layers run."""
    n = len(config["layers"])
    loop = config.get("loop") or {"start": 0, "stop": 0, "times": 0}
    start, stop = loop["start"], loop["stop"]
    order = [(i, None) for i in range(start)]
    for t in range(loop["times"]):
        order += [(i, t if i == start else None) for i in range(start, stop)]
    return order + [(i, None) for i in range(stop, n)]


def forward(config, weights, tokens, streams=None, margins=None):
    """Logits [T, vocab] of one sequence from position 0.  `weights`: {tensor name: float64 array}.
    `streams`, a list, receives the residual stream after every layer run; `margins` the tokens' margins at every mixture and
    every retention."""
    eps, m = config["norm"]["eps"], config["residual_mult"]
    x = weights["embed"][np.asarray(tokens)]
    for i, step in run_order(config):
        layer = config["layers"][i]
        if step is not None:
            x = x + weights["loop.step"][step]
        mix = MIXERS[layer["type"]]
        h, w = rms_norm(x, weights[f"l{i}.norm1"], eps), sub(weights, f"l{i}.mix")
        if layer["type"] == "parallel" and margins is not None:
            margins.append(retention_margin(h, sub(w, "right"), layer["mixer"]["right"]))
        x = x + m * mix(h, w, layer["mixer"], eps)
        mlp = layer.get("mlp")
        if mlp is not None:
            h, w = rms_norm(x, weights[f"l{i}.norm2"], eps), sub(weights, f"l{i}.mlp")
            if mlp["kind"] == "moe" and margins is not None:
                margins.append(route_margin(h, w, mlp))
            x = x + m * (gated_ffn(h, w, relu) if mlp["kind"] == "dense" else moe_ffn(h, w, mlp))
        if streams is not None:
            streams.append(x.copy())
    return rms_norm(x, weights["final.norm"], eps) @ weights["embed"].T


class PlainSagopel:
    """A model folder (config.json, model.safetensors) run by the functions above."""

    def __init__(self, folder):
        import json
        import os

        import torch
        from safetensors.torch import load_file
        with open(os.path.join(folder, "config.json")) as f:
            self.cfg = json.load(f)
        self.tensors = {n: t.to(torch.float64).numpy() for n, t in load_file(os.path.join(folder, "model.safetensors")).items()}

    def logits(self, tokens, want=None):
        rows = forward(self.cfg, self.tensors, tokens)
        return rows if want is None else rows[np.asarray(want, dtype=np.int64)]

    def streams(self, tokens):
        out = []
        forward(self.cfg, self.tensors, tokens, streams=out)
        return np.stack(out)

    def margins(self, tokens):
        """The smallest margin of every token over the mixtures and retentions (None: the model has none)."""
        out = []
        forward(self.cfg, self.tensors, tokens, margins=out)
        return np.min(out, axis=0) if out else None

    def decisive(self, tokens, rng, least=40.0, tries=400):
        """`tokens` with every position that is a close call (a margin below `least`: another choice of experts, or a head of
        retention that nearly cancels) drawn again, until none is left: no comparison with an engine that rounds then
        rests on a close call.  (A position's margins depend on the
        tokens up to it only, so what lies before the first close call stays as it is.)"""
        tokens = list(tokens)
        vocab = self.tensors["embed"].shape[0]
        for _ in range(tries):
            margins = self.margins(tokens)
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
