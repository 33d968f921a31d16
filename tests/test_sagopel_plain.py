"""Pins of the plain Sagopel implementation (tests/plain/sagopel_plain.py) that need no GPU: special cases against
library routines, and properties chosen so that a plausible misreading of a mechanism fails them; then the
configuration class (keys, checks, tensor names) and the rotation table of the engine's position part."""
import copy
import math

import numpy as np
import pytest
import torch

from plain import sagopel_plain as P

RNG = np.random.default_rng(58)


def tensor(a):
    return torch.from_numpy(np.ascontiguousarray(a))


def test_norms_against_the_library():
    x, w = RNG.normal(size=(3, 6)), RNG.normal(size=6)
    np.testing.assert_allclose(P.rms_norm(x, w, 1e-2), torch.nn.functional.rms_norm(tensor(x), (6,), tensor(w), 1e-2).numpy(), rtol=1e-12)
    np.testing.assert_allclose(P.over_rms(np.zeros((1, 4)), 1e-5), 0.0)                  # (eps stands inside the root)
    assert P.over_rms(np.full((1, 4), 1e-2), 1.0)[0, 0] == pytest.approx(1e-2 / math.sqrt(1.0001))


def test_the_first_channels_turn_in_halves_and_the_rest_passes():
    x = np.zeros((1, 1, 10))
    x[0, 0, 1], x[0, 0, 8] = 1.0, 5.0                       # six channels turn: pairs (0,3) (1,4) (2,5)
    angle = 4 * 100.0 ** (-2 / 6)
    y = P.rotate(x, [4], 6, 100.0)
    assert y[0, 0, 1] == pytest.approx(math.cos(angle)) and y[0, 0, 4] == pytest.approx(math.sin(angle))
    assert y[0, 0, 8] == 5.0 and np.count_nonzero(y) == 3
    assert np.array_equal(P.rotate(x, [0], 6, 100.0), x)
    q, k = RNG.normal(size=(1, 1, 8)), RNG.normal(size=(1, 1, 8))
    dot = lambda i, j: float(np.sum(P.rotate(q, [i], 8, 50.0) * P.rotate(k, [j], 8, 50.0)))
    assert dot(9, 4) == pytest.approx(dot(25, 20)) and dot(9, 4) != pytest.approx(dot(4, 9))


def test_the_engines_rotation_table_has_the_same_angles():
    from mini_llm_runtime_amd.config.specs import PositionSpec
    from mini_llm_runtime_amd.parts.rope import RopeSplitHalf
    for dims, base in ((8, 500.0), (2, 9.0), (64, 1e6)):
        table = RopeSplitHalf(PositionSpec("rope_split_half", dims, base)).rotation(50, "cpu").table.double().numpy()
        angle = np.arange(50)[:, None] * base ** (-2.0 * np.arange(dims // 2) / dims)
        np.testing.assert_allclose(table, np.concatenate([np.cos(angle), np.sin(angle)], axis=1), atol=5e-6)


def test_a_window_keeps_the_first_tokens_and_never_looks_ahead():
    seen = P.seen_in_window(np.arange(9), np.arange(9), 3, 2)
    assert [np.nonzero(row)[0].tolist() for row in seen] == [[0], [0, 1], [0, 1, 2], [0, 1, 2, 3], [0, 1, 2, 3, 4], [0, 1, 3, 4, 5], [0, 1, 4, 5, 6],
                                                             [0, 1, 5, 6, 7], [0, 1, 6, 7, 8]]
    assert np.array_equal(P.seen_in_window([5], np.arange(9), 1, 0)[0], np.arange(9) == 5)
    assert np.array_equal(P.seen_in_window([2], np.arange(9), 1, 8)[0], np.arange(9) <= 2)       # more kept than there is


def test_attention_against_the_library_with_scores_capped_before_the_softmax():
    q, k, v = RNG.normal(size=(7, 4, 6)), RNG.normal(size=(7, 2, 6)), RNG.normal(size=(7, 2, 3))
    seen = P.seen_in_window(np.arange(7), np.arange(7), 3, 1)
    want = [torch.nn.functional.scaled_dot_product_attention(tensor(q[:, h])[None], tensor(k[:, h // 2])[None], tensor(v[:, h // 2])[None],
                                                             attn_mask=tensor(seen), scale=0.7)[0].numpy() for h in range(4)]
    np.testing.assert_allclose(P.attend(q, k, v, 0.7, 1e7, seen), np.concatenate(want, axis=1), rtol=1e-9, atol=1e-9)
    assert P.capped(1e9, 30.0) == pytest.approx(30.0) and P.capped(-1e9, 30.0) == pytest.approx(-30.0) and P.capped(1e-4, 30.0) == pytest.approx(1e-4)
    two = P.attend(np.array([[[1.0]], [[50.0]]]), np.array([[[0.0]], [[9.0]]]), np.array([[[0.0]], [[1.0]]]), 1.0, 2.0, P.seen_in_window([0, 1], [0, 1], 2, 0))
    assert two[1, 0] == pytest.approx(1.0 / (1.0 + math.exp(-2.0)))                      # no score beyond the cap


def attention_weights(cfg, width):
    H, G, D, V = cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    return {"q": RNG.normal(size=(H * D, width)), "k": RNG.normal(size=(G * D, width)), "v": RNG.normal(size=(G * V, width)),
            "q.b": RNG.normal(size=H * D), "k.b": RNG.normal(size=G * D), "v.b": RNG.normal(size=G * V), "q.norm": RNG.normal(size=D),
            "k.norm": RNG.normal(size=D), "o": RNG.normal(size=(width, H * V))}


WINDOW = dict(heads=4, kv_heads=2, dim=6, vdim=5, scale=0.4, softcap=9.0, rot=dict(dims=4, base=100.0), mask=dict(size=3, keep_first=2))


def test_biases_come_before_the_norm_and_the_norm_before_the_rotation():
    w, T = attention_weights(WINDOW, 5), 8
    x = RNG.normal(size=(T, 5))
    q = P.rotate(P.rms_norm((x @ w["q"].T + w["q.b"]).reshape(T, 4, 6), w["q.norm"], 1e-5), np.arange(T), 4, 100.0)
    k = P.rotate(P.rms_norm((x @ w["k"].T + w["k.b"]).reshape(T, 2, 6), w["k.norm"], 1e-5), np.arange(T), 4, 100.0)
    v = (x @ w["v"].T + w["v.b"]).reshape(T, 2, 5)
    heads = []
    for h in range(4):
        s = 9.0 * np.tanh(0.4 * q[7, h] @ k[[0, 1, 5, 6, 7], h // 2].T / 9.0)            # what position 7 sees
        heads.append(np.exp(s) / np.exp(s).sum() @ v[[0, 1, 5, 6, 7], h // 2])
    np.testing.assert_allclose(P.window_attention(x, w, WINDOW, 1e-5)[7], w["o"] @ np.concatenate(heads), rtol=1e-9, atol=1e-9)


def test_a_decayed_sum_is_attention_with_powers_of_the_decay():
    q, k, v, T = RNG.normal(size=(9, 4)), RNG.normal(size=(9, 4)), RNG.normal(size=(9, 3)), 9
    for decay in (0.7, 1.0):
        powers = np.tril(decay ** np.maximum(np.arange(T)[:, None] - np.arange(T)[None, :], 0))
        np.testing.assert_allclose(P.decayed_sum(q, k, v, decay), ((q @ k.T) * powers) @ v, rtol=1e-9, atol=1e-9)
    # the token's own write is read by itself, undecayed
    np.testing.assert_allclose(P.decayed_sum(q[:1], k[:1], v[:1], 0.1)[0], float(q[0] @ k[0]) * v[0])


def test_lightning_norms_all_heads_as_one_row_and_retention_each_by_itself():
    width, T = 5, 6
    x = RNG.normal(size=(T, width))
    cfg = dict(heads=2, dim=4, vdim=3, decay=[0.5, 0.9])
    w = {n: RNG.normal(size=s) for n, s in (("q", (8, width)), ("k", (8, width)), ("v", (6, width)), ("g", (6, width)), ("norm", (6,)), ("o", (width, 6)))}
    silu = lambda z: torch.nn.functional.silu(tensor(z)).numpy()
    q, k, v = silu(x @ w["q"].T), silu(x @ w["k"].T), silu(x @ w["v"].T)
    o = np.concatenate([P.decayed_sum(q[:, :4], k[:, :4], v[:, :3], 0.5), P.decayed_sum(q[:, 4:], k[:, 4:], v[:, 3:], 0.9)], axis=1)
    gate = torch.sigmoid(tensor(x @ w["g"].T)).numpy()
    np.testing.assert_allclose(P.lightning(x, w, cfg, 1e-5), (P.rms_norm(o, w["norm"], 1e-5) * gate) @ w["o"].T, rtol=1e-9, atol=1e-10)
    cfg["rot"] = dict(dims=2, base=10.0)
    pos = np.arange(T)
    turned = lambda n: P.rotate((x @ w[n].T).reshape(T, 2, 4), pos, 2, 10.0)
    q, k, v = turned("q"), turned("k") / 2.0, (x @ w["v"].T).reshape(T, 2, 3)             # k over the root of four
    o = np.stack([P.decayed_sum(q[:, h], k[:, h], v[:, h], cfg["decay"][h]) for h in range(2)], axis=1)
    o = (o / np.sqrt((o * o).mean(axis=2, keepdims=True) + 1e-5)).reshape(T, 6)
    np.testing.assert_allclose(P.retention(x, w, cfg, 1e-5), (o * silu(x @ w["g"].T)) @ w["o"].T, rtol=1e-9, atol=1e-10)


def test_the_choice_is_corrected_and_the_weights_are_not():
    z = np.array([[2.0, 1.0, 0.0, -1.0]])
    s = torch.softmax(tensor(z[0]), dim=0).numpy()
    w = dict(router=z.T, correction=np.array([-1.0, 0.0, 0.0, 0.6]))
    ids, weights = P.route(np.ones((1, 1)), w, dict(experts=3, identity=1, top=2))
    assert ids[0].tolist() == [3, 1]
    np.testing.assert_allclose(weights[0], s[[3, 1]], rtol=1e-12)                         # as they are, over all four
    assert np.all(np.isinf(P.route_margin(np.ones((1, 1)), w, dict(router=dict(experts=3, identity=1, top=4)))))


def test_identities_give_the_input_back_and_the_shared_expert_joins_every_token():
    width, ff = 4, 3
    w = {"router": RNG.normal(size=(5, width)), "correction": np.array([0.0, 0.0, 0.0, 0.3, 0.3])}
    for e in ("e0", "e1", "e2", "shared"):
        w.update({f"{e}.gate": RNG.normal(size=(ff, width)), f"{e}.up": RNG.normal(size=(ff, width)), f"{e}.down": RNG.normal(size=(width, ff))})
    cfg = dict(kind="moe", expert=dict(ff=ff), shared=dict(ff=ff), router=dict(experts=3, identity=2, top=3))
    x = RNG.normal(size=(5, width))
    ids, weights = P.route(x, w, cfg["router"])
    assert (ids >= 3).any() and (ids < 3).any()

    def expert(name, row):
        g = w[name + ".gate"] @ row
        return w[name + ".down"] @ (g / (1.0 + np.exp(-g)) * (w[name + ".up"] @ row))
    for t in range(5):
        want = sum(a * (x[t] if e >= 3 else expert(f"e{e}", x[t])) for e, a in zip(ids[t], weights[t])) + expert("shared", x[t])
        np.testing.assert_allclose(P.moe_ffn(x, w, cfg)[t], want, rtol=1e-9)


def small_config():
    left = dict(WINDOW, dim=8, vdim=6)
    right = dict(heads=3, dim=4, vdim=10, decay=[0.9, 0.99, 1.0], rot=dict(dims=2, base=7.0))
    light = dict(type="lightning", mixer=dict(heads=2, dim=6, vdim=4, decay=[0.5, 0.8]), mlp=dict(kind="dense", ff=9))
    moe = dict(kind="moe", expert=dict(ff=10), shared=dict(ff=7), router=dict(experts=4, identity=2, top=3))
    return dict(architecture="Sagopel", vocab=19, width=12, norm=dict(eps=1e-5), residual_mult=0.6, loop=dict(start=1, stop=2, times=3),
                layers=[light, dict(type="parallel", mixer=dict(left=left, right=right), mlp=moe), dict(light, mlp=None)])


def test_looped_passes_start_with_a_vector_and_every_sublayer_joins_with_the_factor():
    from mini_llm_runtime_amd.config import config_from_dict
    from mini_llm_runtime_amd.parts import expected_tensors
    from mini_llm_runtime_amd.weights import random_tensors
    cfg = small_config()
    w = {n: t.double().numpy() for n, t in random_tensors(expected_tensors(config_from_dict(cfg)), 5, matrix_std=0.3).items() if n != "head"}
    tokens = [3, 1, 4, 1, 5, 9, 2, 6]
    streams = []
    logits = P.forward(cfg, w, tokens, streams=streams)
    assert len(streams) == 5 and logits.shape == (8, 19)
    x = w["embed"][np.asarray(tokens)]
    x = x + 0.6 * P.lightning(P.rms_norm(x, w["l0.norm1"], 1e-5), P.sub(w, "l0.mix"), cfg["layers"][0]["mixer"], 1e-5)
    h = P.rms_norm(x, w["l0.norm2"], 1e-5)
    x = x + 0.6 * (np.maximum(h @ w["l0.mlp.gate"].T, 0.0) * (h @ w["l0.mlp.up"].T)) @ w["l0.mlp.down"].T
    np.testing.assert_allclose(streams[0], x, rtol=1e-9, atol=1e-12)
    for t in range(3):
        x = x + w["loop.step"][t]
        h, mixer = P.rms_norm(x, w["l1.norm1"], 1e-5), cfg["layers"][1]["mixer"]
        left = P.window_attention(h, P.sub(w, "l1.mix.left"), mixer["left"], 1e-5)
        right = P.retention(h, P.sub(w, "l1.mix.right"), mixer["right"], 1e-5)
        x = x + 0.3 * (P.rms_norm(left, w["l1.mix.left.out"], 1e-5) + P.rms_norm(right, w["l1.mix.right.out"], 1e-5))
        x = x + 0.6 * P.moe_ffn(P.rms_norm(x, w["l1.norm2"], 1e-5), P.sub(w, "l1.mlp"), cfg["layers"][1]["mlp"])
        np.testing.assert_allclose(streams[1 + t], x, rtol=1e-9, atol=1e-12)
    np.testing.assert_allclose(logits, P.rms_norm(streams[4], w["final.norm"], 1e-5) @ w["embed"].T, rtol=1e-9, atol=1e-12)
    np.testing.assert_allclose(P.forward(cfg, w, tokens[:5])[4], logits[4], rtol=1e-9, atol=1e-12)     # what follows does not matter


def test_configuration_names_every_tensor():
    from mini_llm_runtime_amd.config import config_from_dict
    from mini_llm_runtime_amd.parts import expected_tensors
    cfg = config_from_dict(small_config())
    assert cfg.to_dict() == small_config() and config_from_dict(cfg.to_dict()) == cfg
    spec = cfg.model_spec()
    assert [(r.layer, r.cache, r.add_vector) for r in spec.schedule] == [(0, 0, None), (1, 1, 0), (1, 2, 1), (1, 3, 2), (2, 4, None)]
    assert [layer.residual_scale for layer in spec.layers] == [0.6] * 3 and spec.layers[2].ffn is None
    shapes = {"embed": (19, 12), "final.norm": (12,), "loop.step": (3, 12), "l0.norm1": (12,), "l0.norm2": (12,), "l1.norm1": (12,), "l1.norm2": (12,),
              "l2.norm1": (12,), "l0.mlp.gate": (9, 12), "l0.mlp.up": (9, 12), "l0.mlp.down": (12, 9)}
    for i in (0, 2):
        shapes.update({f"l{i}.mix.q": (12, 12), f"l{i}.mix.k": (12, 12), f"l{i}.mix.v": (8, 12), f"l{i}.mix.g": (8, 12), f"l{i}.mix.norm": (8,),
                       f"l{i}.mix.o": (12, 8)})
    shapes.update({"l1.mix.left.q": (32, 12), "l1.mix.left.k": (16, 12), "l1.mix.left.v": (12, 12), "l1.mix.left.q.b": (32,), "l1.mix.left.k.b": (16,),
                   "l1.mix.left.v.b": (12,), "l1.mix.left.q.norm": (8,), "l1.mix.left.k.norm": (8,), "l1.mix.left.o": (12, 24), "l1.mix.left.out": (12,),
                   "l1.mix.right.q": (12, 12), "l1.mix.right.k": (12, 12), "l1.mix.right.v": (30, 12), "l1.mix.right.g": (30, 12),
                   "l1.mix.right.o": (12, 30), "l1.mix.right.out": (12,), "l1.mlp.router": (6, 12), "l1.mlp.correction": (6,),
                   "l1.mlp.shared.gate": (7, 12), "l1.mlp.shared.up": (7, 12), "l1.mlp.shared.down": (12, 7)})
    for e in range(4):
        shapes.update({f"l1.mlp.e{e}.gate": (10, 12), f"l1.mlp.e{e}.up": (10, 12), f"l1.mlp.e{e}.down": (12, 10)})
    named = {n: tuple(t.shape) for n, t in expected_tensors(cfg).items() if not t.optional}
    assert named == shapes                                                                # these and no others
    plain_order = small_config()
    plain_order.pop("loop")
    cfg = config_from_dict(plain_order)
    assert cfg.to_dict() == plain_order and "loop.step" not in expected_tensors(cfg)
    assert [(r.layer, r.add_vector) for r in cfg.model_spec().schedule] == [(0, None), (1, None), (2, None)]


def test_configuration_refuses_what_it_cannot_mean():
    from mini_llm_runtime_amd.config import ConfigError, config_from_dict

    def broken(change):
        cfg = copy.deepcopy(small_config())
        change(cfg)
        with pytest.raises(ConfigError):
            config_from_dict(cfg)
    left, right = (lambda c: c["layers"][1]["mixer"]["left"]), (lambda c: c["layers"][1]["mixer"]["right"])
    broken(lambda c: left(c).update(heads=3))                                    # no multiple of kv_heads
    broken(lambda c: left(c)["rot"].update(dims=3))                              # odd
    broken(lambda c: left(c)["rot"].update(dims=10))                             # more than a head has
    broken(lambda c: right(c)["rot"].update(dims=6))
    broken(lambda c: left(c).update(softcap=0.0))
    broken(lambda c: left(c)["mask"].update(size=0))
    broken(lambda c: left(c)["mask"].update(keep_first=-1))
    broken(lambda c: left(c).pop("scale"))
    broken(lambda c: right(c).pop("rot"))
    broken(lambda c: right(c).update(decay=[0.5]))                               # not one a head
    broken(lambda c: c["layers"][0]["mixer"].update(decay=[0.5, 0.0]))
    broken(lambda c: c["layers"][1]["mixer"].pop("right"))
    broken(lambda c: c["layers"][1].update(type="attention"))
    broken(lambda c: c["layers"][1]["mlp"]["router"].update(top=7))              # more choices than outputs
    broken(lambda c: c["layers"][1]["mlp"]["router"].update(identity=-1))
    broken(lambda c: c["layers"][1]["mlp"].pop("expert"))
    broken(lambda c: c["layers"][0]["mlp"].update(kind="gated"))
    broken(lambda c: c["loop"].update(start=3, stop=2))
    broken(lambda c: c["loop"].update(times=0))
    broken(lambda c: c["loop"].update(stop=4))
    broken(lambda c: c.update(layers=[]))
    broken(lambda c: c.pop("norm"))


def test_a_mixture_without_identities_or_a_shared_expert():
    from mini_llm_runtime_amd.config import config_from_dict
    from mini_llm_runtime_amd.parts import expected_tensors
    cfg = small_config()
    cfg["layers"][1]["mlp"] = dict(kind="moe", expert=dict(ff=10), router=dict(experts=4, top=4))
    names = expected_tensors(config_from_dict(cfg))
    assert names["l1.mlp.router"].shape == (4, 12) and not any(".shared." in n for n in names)
