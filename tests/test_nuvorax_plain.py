"""Pins of the plain Nuvorax implementation (tests/plain/nuvorax_plain.py) that need no GPU: special cases against
library routines, and properties chosen so that a plausible misreading of a mechanism fails them; then the
configuration class (keys, checks, tensor names) and the rotation table of the engine's position part."""
import copy
import math

import numpy as np
import pytest
import torch

from plain import nuvorax_plain as P

RNG = np.random.default_rng(57)


def tensor(a):
    return torch.from_numpy(np.ascontiguousarray(a))


def test_the_norm_takes_the_mean_off_and_has_no_bias():
    x, w = RNG.normal(size=(4, 10)) + 3.0, RNG.normal(size=10)
    want = torch.nn.functional.layer_norm(tensor(x), (10,), tensor(w), None, 1e-3).numpy()
    np.testing.assert_allclose(P.layer_norm(x, w, 1e-3), want, rtol=1e-12, atol=1e-12)
    np.testing.assert_allclose(P.layer_norm(np.full((1, 4), 7.0), np.ones(4), 1e-5), 0.0)


def test_head_norm_against_the_library():
    x, w = RNG.normal(size=(3, 2, 6)), RNG.normal(size=6)
    want = torch.nn.functional.rms_norm(tensor(x), (6,), tensor(w), 1e-3).numpy()
    np.testing.assert_allclose(P.rms_norm(x, w, 1e-3), want, rtol=1e-12)


def test_keys_turn_in_halves_of_the_rotated_extent_and_the_rest_passes():
    x = np.zeros((1, 1, 10))
    x[0, 0, 1], x[0, 0, 8] = 1.0, 5.0                       # six channels turn: pairs (0,3) (1,4) (2,5)
    angle = 4 * 100.0 ** (-2 / 6)
    y = P.rotate_keys(x, [4], dict(dims=6, base=100.0))
    assert y[0, 0, 1] == pytest.approx(math.cos(angle)) and y[0, 0, 4] == pytest.approx(math.sin(angle))
    assert y[0, 0, 8] == 5.0 and np.count_nonzero(y) == 3
    assert np.array_equal(P.rotate_keys(x, [0], dict(dims=6, base=100.0)), x)


def test_frequency_bands_keep_fast_pairs_and_slow_the_others():
    sc = dict(factor=8.0, low=1.0, high=4.0, original=100)
    of = lambda wavelength: P.banded_frequencies([2 * math.pi / wavelength], sc)[0] * wavelength / (2 * math.pi)
    assert of(24.9) == pytest.approx(1.0, abs=1e-12)                                  # shorter than original / high: as it is
    assert of(100.1) == pytest.approx(1.0 / 8.0, abs=1e-12)                           # longer than original / low: divided
    assert of(40.0) == pytest.approx(0.5 / 8.0 + 0.5)       # 100 / 40 = 2.5 lies half way between 1 and 4
    assert of(25.0) == pytest.approx(1.0) and of(100.0) == pytest.approx(1.0 / 8.0)      # no jump at the borders
    assert of(30.0) > of(60.0) > of(90.0)


def test_the_engines_rotation_table_has_the_same_angles():
    from mini_llm_runtime_amd.config.specs import FrequencyBands, PositionSpec
    from mini_llm_runtime_amd.parts.rope import Rope
    for dims, base, sc in ((8, 500.0, dict(factor=4.0, low=1.0, high=3.0, original=40)), (20, 1e4, dict(factor=3.0, low=2.0, high=2.0, original=90)),
                           (64, 1e6, dict(factor=16.0, low=0.5, high=9.0, original=3000))):
        table = Rope(PositionSpec("rope", dims, base, bands=FrequencyBands(**sc))).rotation(50, "cpu").table
        if sc["low"] == sc["high"]:                         # (an empty band between: the plain form has nothing to divide by)
            turns = sc["original"] * P.plain_frequencies(dims, base) / (2 * math.pi)
            freq = np.where(turns > sc["high"], 1.0, 1.0 / sc["factor"]) * P.plain_frequencies(dims, base)
        else:
            freq = P.banded_frequencies(P.plain_frequencies(dims, base), sc)
        angles = np.arange(50)[:, None] * freq
        np.testing.assert_allclose(table.double().numpy(), np.concatenate([np.cos(angles), np.sin(angles)], axis=1), atol=4e-6)


def test_turned_values_come_back_as_functions_of_the_distance():
    v = RNG.normal(size=(6, 2, 8))
    pos = np.arange(6)
    np.testing.assert_allclose(P.rotate_values(P.rotate_values(v, pos, 50.0), pos, 50.0, -1.0), v, atol=1e-12)
    # a value read from position 9 that lies at 4 arrives as the same value read from 25 that lies at 20 does
    read = lambda i, j: P.rotate_values(P.rotate_values(v[:1], [j], 50.0), [i], 50.0, -1.0)
    np.testing.assert_allclose(read(9, 4), read(25, 20), atol=1e-12)
    assert not np.allclose(read(9, 4), read(4, 9))
    # pair m is (m, m + half) and turns by base^(-2m / size)
    one = np.zeros((1, 1, 8))
    one[0, 0, 1] = 1.0
    y = P.rotate_values(one, [3], 50.0)
    assert y[0, 0, 1] == pytest.approx(math.cos(3 * 50.0 ** (-2 / 8))) and y[0, 0, 5] == pytest.approx(math.sin(3 * 50.0 ** (-2 / 8)))


def test_the_softmax_has_one_more_summand_that_brings_nothing():
    s = RNG.normal(size=(3, 5)) * 4
    seen = np.ones((3, 5), dtype=bool)
    with_zero = torch.softmax(tensor(np.concatenate([s, np.zeros((3, 1))], axis=1)), dim=1).numpy()[:, :5]
    np.testing.assert_allclose(P.softmax_plus_one(s, seen), with_zero, rtol=1e-12)
    seen[1, 2:] = False
    p = P.softmax_plus_one(s, seen)
    assert np.all(p[1, 2:] == 0.0) and p[1].sum() < 1.0
    np.testing.assert_allclose(P.softmax_plus_one(np.full((1, 1), -800.0), np.ones((1, 1), dtype=bool)), 0.0)
    np.testing.assert_allclose(P.softmax_plus_one(np.full((1, 1), 800.0), np.ones((1, 1), dtype=bool)), 1.0)


def test_scores_are_capped_before_the_softmax():
    assert P.capped(1e9, 30.0) == pytest.approx(30.0) and P.capped(-1e9, 30.0) == pytest.approx(-30.0)
    assert P.capped(1e-4, 30.0) == pytest.approx(1e-4)


def attention_weights(cfg, width):
    H, G, D, V = cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    return {"q": RNG.normal(size=(H * D, width)), "k": RNG.normal(size=(G * D, width)), "v": RNG.normal(size=(G * V, width)),
            "q.norm": RNG.normal(size=D), "k.norm": RNG.normal(size=D), "talk": RNG.normal(size=(H, H)), "g": RNG.normal(size=(H, width)),
            "o": RNG.normal(size=(width, H * V))}


def test_attention_head_by_head_against_the_library():
    """Head g's weights meet the values of head h's kv head, whatever kv head g reads: every (g, h) pair by the library's
    attention with a key of score 0 and a value of 0 in front, the shares added by `talk`."""
    cfg = dict(heads=4, kv_heads=2, dim=6, vdim=4, scale=0.7, softcap=1e6, rot=dict(dims=4, base=100.0))
    width, T = 5, 9
    x, pos = RNG.normal(size=(T, width)), np.arange(T)
    w = attention_weights(cfg, width)
    got = P.attention(x, w, cfg, 1e-5)
    q = P.rotate_keys(P.rms_norm((x @ w["q"].T).reshape(T, 4, 6), w["q.norm"], 1e-5), pos, cfg["rot"])
    k = P.rotate_keys(P.rms_norm((x @ w["k"].T).reshape(T, 2, 6), w["k.norm"], 1e-5), pos, cfg["rot"])
    v = P.rotate_values((x @ w["v"].T).reshape(T, 2, 4), pos, 100.0)
    seen = np.concatenate([np.ones((T, 1), dtype=bool), np.tril(np.ones((T, T), dtype=bool))], axis=1)
    first = lambda a: np.concatenate([np.zeros((1, a.shape[1])), a])
    heads = []
    for h in range(4):
        o = sum(w["talk"][h, g] * torch.nn.functional.scaled_dot_product_attention(
            tensor(q[:, g])[None], tensor(first(k[:, g // 2]))[None], tensor(first(v[:, h // 2]))[None], attn_mask=tensor(seen),
            scale=0.7)[0].numpy() for g in range(4))
        o = P.rotate_values(o[:, None], pos, 100.0, -1.0)[:, 0]
        heads.append(o * torch.sigmoid(tensor(x @ w["g"][h])).numpy()[:, None])
    np.testing.assert_allclose(got, np.concatenate(heads, axis=1) @ w["o"].T, rtol=1e-7, atol=1e-8)


def test_mixing_goes_from_the_second_index_to_the_first():
    p = RNG.random(size=(2, 3, 3))
    talk = np.array([[0.0, 2.0], [0.0, 0.0]])               # head 0 takes head 1's weights twice, head 1 nothing
    mixed = P.mixed_heads(p, talk)
    np.testing.assert_allclose(mixed[0], 2.0 * p[1])
    assert not mixed[1].any()
    np.testing.assert_allclose(P.mixed_heads(p, np.eye(2)), p)


def test_the_first_token_is_one_key_beside_the_sink():
    cfg = dict(heads=1, kv_heads=1, dim=2, vdim=2, scale=1.0, softcap=3.0, rot=dict(dims=2, base=10.0))
    w = attention_weights(cfg, 4)
    x = RNG.normal(size=(1, 4))
    q, k = (P.rms_norm(x @ w[n].T, w[n + ".norm"], 1e-5)[0] for n in "qk")
    s = 3.0 * math.tanh(float(q @ k) / 3.0)
    share = math.exp(s) / (1.0 + math.exp(s)) * w["talk"][0, 0] / (1.0 + math.exp(-float(x[0] @ w["g"][0])))
    np.testing.assert_allclose(P.attention(x, w, cfg, 1e-5)[0], w["o"] @ (share * (w["v"] @ x[0])), rtol=1e-9)


def test_gelu_is_the_exact_one():
    z = np.linspace(-5, 5, 41)
    np.testing.assert_allclose(P.gelu_erf(z), torch.nn.functional.gelu(tensor(z), approximate="none").numpy(), atol=1e-12)
    assert not np.allclose(P.gelu_erf(z), torch.nn.functional.gelu(tensor(z), approximate="tanh").numpy(), atol=1e-6)


def test_an_experts_gate_is_clamped_above_and_its_up_on_both_sides():
    one = np.ones((1, 1))
    y = lambda x, g, u, limit: float(P.clamped_glu(np.array([[x]]), one * g, one * u, one, limit)[0, 0])
    act = lambda g: g / (1.0 + math.exp(-1.702 * g))
    assert y(1.0, 9.0, 0.0, 2.0) == pytest.approx(act(2.0))            # the gate stops at the limit
    assert y(1.0, -9.0, 0.0, 2.0) == pytest.approx(act(-9.0))          # and not below
    assert y(1.0, 1.0, 9.0, 2.0) == pytest.approx(act(1.0) * 3.0)      # up stops at the limit, then one is added
    assert y(1.0, 1.0, -9.0, 2.0) == pytest.approx(-act(1.0))


def test_groups_are_ranked_by_their_best_expert_and_weights_are_softmax_shares():
    z = np.array([[3.0, -9.0, 2.9, 2.8, 0.0, 0.0]])          # groups of two: the first has the best expert, the second the best sum
    w = dict(router=z.T)
    router = dict(experts=6, top=2, scale=1.5, groups=dict(count=3, keep=1))
    ids, weights = P.route(np.ones((1, 1)), w, router)
    assert ids[0].tolist() == [0, 1]
    s = torch.softmax(tensor(z[0]), dim=0).numpy()            # over ALL experts; the chosen ones' shares of their sum
    np.testing.assert_allclose(weights[0], s[[0, 1]] / s[[0, 1]].sum() * 1.5)
    ids, weights = P.route(np.ones((1, 1)), w, dict(router, groups=dict(count=3, keep=2)))
    assert ids[0].tolist() == [0, 2] and weights[0].sum() == pytest.approx(1.5)
    assert P.route(np.ones((1, 1)), w, dict(router, top=6, groups=dict(count=1, keep=1)))[0][0].tolist() == [0, 2, 3, 4, 5, 1]
    margins = P.route_margin(RNG.normal(size=(5, 4)), dict(router=RNG.normal(size=(6, 4))), dict(experts=6, top=6))
    assert np.all(np.isinf(margins))


def test_the_mixture_adds_a_shared_expert_behind_one_gate_a_token():
    width, ff = 4, 3
    w = {"router": RNG.normal(size=(4, width)), "shared.sg": RNG.normal(size=(1, width))}
    for e in ("e0", "e1", "e2", "e3", "shared"):
        w.update({f"{e}.gate": RNG.normal(size=(ff, width)), f"{e}.up": RNG.normal(size=(ff, width)), f"{e}.down": RNG.normal(size=(width, ff))})
    cfg = dict(kind="moe", expert=dict(ff=ff, limit=0.6), shared=dict(ff=ff, limit=1.2),
               router=dict(experts=4, top=2, scale=1.3, groups=dict(count=2, keep=2)))
    x = RNG.normal(size=(5, width))
    ids, weights = P.route(x, w, cfg["router"])

    def expert(name, row, limit):
        g, u = np.minimum(w[name + ".gate"] @ row, limit), np.clip(w[name + ".up"] @ row, -limit, limit)
        return w[name + ".down"] @ (g / (1.0 + np.exp(-1.702 * g)) * (u + 1.0))
    for t in range(5):
        want = sum(a * expert(f"e{e}", x[t], 0.6) for e, a in zip(ids[t], weights[t]))
        want = want + expert("shared", x[t], 1.2) / (1.0 + math.exp(-float(w["shared.sg"][0] @ x[t])))
        np.testing.assert_allclose(P.moe_ffn(x, w, cfg)[t], want, rtol=1e-9)


def small_config():
    mixer = dict(heads=4, kv_heads=2, dim=8, vdim=6, scale=0.3, softcap=20.0,
                 rot=dict(base=100.0, dims=4, scaling=dict(factor=4.0, low=1.0, high=3.0, original=30)))
    other = dict(heads=3, kv_heads=3, dim=4, vdim=4, scale=0.5, softcap=9.0, rot=dict(base=7.0, dims=4))
    moe = dict(kind="moe", expert=dict(ff=10, limit=0.8), shared=dict(ff=7, limit=1.6),
               router=dict(experts=4, top=2, scale=1.5, groups=dict(count=2, keep=1)))
    return dict(architecture="Nuvorax", vocab=19, width=12, norm=dict(eps=1e-5), embedding=dict(scale=2.5), logit_scale=0.5,
                layers=[dict(type="attention", mixer=mixer, mlp=moe), dict(type="attention", mixer=other, mlp=None),
                        dict(type="attention", mixer=mixer, mlp=dict(kind="dense", ff=9))])


def test_both_sublayers_read_the_one_norm_and_the_ends_have_factors():
    from mini_llm_runtime_amd.config import config_from_dict
    from mini_llm_runtime_amd.parts import expected_tensors
    from mini_llm_runtime_amd.weights import random_tensors
    cfg = small_config()
    w = {n: t.double().numpy() for n, t in random_tensors(expected_tensors(config_from_dict(cfg)), 5, matrix_std=0.3).items()}
    tokens = [3, 1, 4, 1, 5, 9, 2, 6]
    streams = []
    logits = P.forward(cfg, w, tokens, streams=streams)
    assert len(streams) == 3 and logits.shape == (8, 19)
    x = w["embed"][np.asarray(tokens)] * 2.5
    h = P.layer_norm(x, w["l0.norm1"], 1e-5)
    side = P.attention(h, P.layer_weights(w, 0, "mix"), cfg["layers"][0]["mixer"], 1e-5) + P.moe_ffn(h, P.layer_weights(w, 0, "mlp"), cfg["layers"][0]["mlp"])
    np.testing.assert_allclose(streams[0], x + side, rtol=1e-9, atol=1e-12)
    h = P.layer_norm(streams[1], w["l2.norm1"], 1e-5)
    side = P.attention(h, P.layer_weights(w, 2, "mix"), cfg["layers"][2]["mixer"], 1e-5) + P.gelu_erf(h @ w["l2.mlp.up"].T) @ w["l2.mlp.down"].T
    np.testing.assert_allclose(streams[2], streams[1] + side, rtol=1e-9, atol=1e-12)
    np.testing.assert_allclose(logits, P.layer_norm(streams[2], w["final.norm"], 1e-5) @ w["head"].T * 0.5, rtol=1e-9, atol=1e-12)
    np.testing.assert_allclose(P.forward(cfg, w, tokens[:5])[4], logits[4], rtol=1e-9, atol=1e-12)     # what follows does not matter


def test_configuration_names_every_tensor():
    from mini_llm_runtime_amd.config import config_from_dict
    from mini_llm_runtime_amd.parts import expected_tensors
    cfg = config_from_dict(small_config())
    assert cfg.to_dict() == small_config() and config_from_dict(cfg.to_dict()) == cfg
    spec = cfg.model_spec()
    assert [(r.layer, r.cache) for r in spec.schedule] == [(0, 0), (1, 1), (2, 2)]
    assert spec.embed.scale == 2.5 and spec.head.scale == 0.5 and spec.layers[1].mixer.position.bands is None
    names = expected_tensors(cfg)
    shapes = {"embed": (19, 12), "head": (19, 12), "final.norm": (12,), "l0.norm1": (12,), "l1.norm1": (12,), "l2.norm1": (12,)}
    for i, (q, k, v, d, heads) in ((0, (32, 16, 12, 8, 4)), (1, (12, 12, 12, 4, 3)), (2, (32, 16, 12, 8, 4))):
        shapes.update({f"l{i}.mix.q": (q, 12), f"l{i}.mix.k": (k, 12), f"l{i}.mix.v": (v, 12), f"l{i}.mix.q.norm": (d,), f"l{i}.mix.k.norm": (d,),
                       f"l{i}.mix.talk": (heads, heads), f"l{i}.mix.g": (heads, 12), f"l{i}.mix.o": (12, heads * v // (2 if heads == 4 else 3))})
    shapes.update({"l0.mlp.router": (4, 12), "l0.mlp.shared.gate": (7, 12), "l0.mlp.shared.up": (7, 12), "l0.mlp.shared.down": (12, 7),
                   "l0.mlp.shared.sg": (1, 12), "l2.mlp.up": (9, 12), "l2.mlp.down": (12, 9)})
    for e in range(4):
        shapes.update({f"l0.mlp.e{e}.gate": (10, 12), f"l0.mlp.e{e}.up": (10, 12), f"l0.mlp.e{e}.down": (12, 10)})
    assert {n: tuple(t.shape) for n, t in names.items()} == shapes                # these and no others


def test_configuration_refuses_what_it_cannot_mean():
    from mini_llm_runtime_amd.config import ConfigError, config_from_dict

    def broken(change):
        cfg = copy.deepcopy(small_config())
        change(cfg)
        with pytest.raises(ConfigError):
            config_from_dict(cfg)
    broken(lambda c: c["layers"][0]["mixer"].update(heads=3))                    # no multiple of kv_heads
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=3))              # odd
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=10))             # more than a head has
    broken(lambda c: c["layers"][0]["mixer"].update(vdim=5))                     # values turn in pairs
    broken(lambda c: c["layers"][0]["mixer"].update(softcap=0.0))
    broken(lambda c: c["layers"][0]["mixer"].pop("scale"))
    broken(lambda c: c["layers"][0]["mixer"].pop("rot"))
    broken(lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(high=0.5))     # below low
    broken(lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("original"))
    broken(lambda c: c["layers"][1].update(type="latent_attention"))
    broken(lambda c: c["layers"][0]["mlp"]["router"].update(top=3))              # more choices than the kept groups hold
    broken(lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=3))  # no equal groups
    broken(lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(keep=3))
    broken(lambda c: c["layers"][0]["mlp"]["expert"].update(limit=0.0))
    broken(lambda c: c["layers"][2]["mlp"].update(kind="gated"))
    broken(lambda c: c.update(layers=[]))
    broken(lambda c: c.pop("norm"))
