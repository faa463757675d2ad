"""CPU: the Lebelix oracle against closed forms, that the small test models react to every mechanism (so that a parity test on them can
fail), the configuration reader and the layout of the weights."""
import json

import lebelix_cases as cases
import numpy as np
import pytest

from oracle import lebelix_oracle as orc
from skainet_amd import hybrid, lebelix, models


def test_norms_and_activations_known_values():
    x = np.array([[3.0, -4.0]])
    assert np.allclose(orc.offset_norm(x, np.array([0.0, 1.0]), 0.0), [[3 / np.sqrt(12.5), -8 / np.sqrt(12.5)]])
    assert np.allclose(orc.plain_norm(x, np.array([0.0, 1.0]), 0.0), [[0.0, -4 / np.sqrt(12.5)]])
    assert np.allclose(orc.unit(np.array([3.0, 4.0])), [0.6, 0.8], atol=1e-7)
    assert orc.gelu_tanh(np.array(0.0)) == 0.0
    assert np.isclose(orc.gelu_tanh(np.array(1.0)), 0.841192, atol=1e-6) and np.isclose(orc.gelu_tanh(np.array(-1.0)), -0.158808, atol=1e-6)


def test_rotation_of_a_part():
    x = np.arange(1.0, 7.0)[None].repeat(3, 0)
    y = orc.rotate_half(x, [0, 1, 7], 100.0, 4)
    assert np.allclose(y[0], x[0]) and np.allclose(y[:, 4:], x[:, 4:])
    for i, f in ((0, 1.0), (1, 0.1)):
        c, s = np.cos(7 * f), np.sin(7 * f)
        assert np.allclose(y[2, [i, i + 2]], [x[2, i] * c - x[2, i + 2] * s, x[2, i + 2] * c + x[2, i] * s])


def test_masks():
    w, c = orc.window_mask(6, 2), orc.chunk_mask(7, 3)
    assert np.array_equal(np.flatnonzero(w[4]), [3, 4]) and np.array_equal(np.flatnonzero(w[0]), [0])
    assert np.array_equal(np.flatnonzero(c[5]), [3, 4, 5]) and np.array_equal(np.flatnonzero(c[6]), [6]) and np.array_equal(np.flatnonzero(c[2]), [0, 1, 2])


def test_softmax_with_a_sink():
    s, m = np.array([[1.0, 5.0, -2.0]]), np.array([[True, False, True]])
    e = np.exp([1.0, -2.0])
    assert np.allclose(orc.sink_softmax(s, m)[0, [0, 2]], e / (1 + e.sum())) and orc.sink_softmax(s, m)[0, 1] == 0
    assert np.allclose(orc.sink_softmax(s - 2000, m), 0) and np.allclose(orc.sink_softmax(s + 2000, m).sum(), 1)
    assert np.allclose(orc.softmax(s, m)[0, [0, 2]], e / e.sum())


def test_convolution():
    x, taps = np.array([[1.0], [2.0], [4.0]]), np.array([[100.0, 10.0, 1.0]])
    assert np.allclose(orc.causal_conv(x, taps)[:, 0], [1, 12, 124])


def test_gated_delta_rule_special_cases():
    rng = np.random.default_rng(1)
    q, k, v = (rng.standard_normal((6, 1, 3)) for _ in range(3))
    k = orc.unit(k)
    one, rate = np.ones((6, 1, 3)), np.ones((6, 1))
    o, S = orc.gated_delta_rule(k, k, v, one, rate)  # full rate: what is read at the key just written is the value
    assert np.allclose(o, v, atol=1e-5)
    o, _ = orc.gated_delta_rule(q, k, v, 0 * one, rate)  # everything forgotten: only the token itself
    assert np.allclose(o[:, 0], (q[:, 0] * k[:, 0]).sum(1)[:, None] * v[:, 0])
    a = orc.gated_delta_rule(q, k, v, 0.7 * one, 0.4 * rate)
    first, state = orc.gated_delta_rule(q[:2], k[:2], v[:2], 0.7 * one[:2], 0.4 * rate[:2])
    rest, state = orc.gated_delta_rule(q[2:], k[2:], v[2:], 0.7 * one[2:], 0.4 * rate[2:], state)
    assert np.allclose(np.concatenate([first, rest]), a[0]) and np.allclose(state, a[1])


def _window(f):
    return lambda T, size: f(T, size + 1)


MUTATIONS = {
    "weights of the norm around one": ("offset_norm", lambda f: lambda x, w, eps: f(x, w - 1.0, eps)),
    "no unit keys": ("unit", lambda f: lambda x: x),
    "no rotation": ("rotate_half", lambda f: lambda x, p, base, dims: x),
    "positions from 1 in one place": ("latent_row", lambda f: lambda h, w, pre, m, eps: (f(h, w, pre, m, eps)[0], np.roll(f(h, w, pre, m, eps)[1], 1, axis=0))),
    "window one longer": ("window_mask", _window),
    "chunk one longer": ("chunk_mask", _window),
    "no cap": ("soft_cap", lambda f: lambda s, cap: s),
    "no sink": ("sink_softmax", lambda f: orc.softmax),
    "convolution one token late": ("causal_conv", lambda f: lambda x, taps: f(np.concatenate([0 * x[:1], x[:-1]]), taps)),
    "no decay": ("channel_decay", lambda f: lambda z, a, b: np.ones_like(z)),
    "one decay per head": ("channel_decay", lambda f: lambda z, a, b: np.broadcast_to(f(z, a, b).mean(-1, keepdims=True), z.shape)),
    "nothing from the side table": ("token_side", lambda f: lambda x, *a: 0 * x),
    "activation linear": ("gelu_tanh", lambda f: lambda z: z),
}


@pytest.mark.parametrize("what", sorted(MUTATIONS))
def test_the_models_react_to_every_mechanism(what, monkeypatch):
    cfg, *ranks = cases.MODELS["mixed"]
    w = cases.weights(cfg, *ranks)
    toks = cases.tokens(cfg, 80)
    want = orc.forward(cfg, w, toks)
    name, mutate = MUTATIONS[what]
    monkeypatch.setattr(orc, name, mutate(getattr(orc, name)))
    err = cases.logit_error(orc.forward(cfg, w, toks), want)
    assert np.quantile(err, 0.8) > 1.5 * cases.TOLERANCE["bfloat16"], err
    assert err[40:].max() > 100 * cases.TOLERANCE["float32"]


def test_latents_come_from_the_layer_that_is_named():
    cfg, *ranks = cases.MODELS["mixed"]
    w, toks = cases.weights(cfg, *ranks), cases.tokens(cfg, 50)
    want, loud = orc.forward(cfg, w, toks), {k: (1.5 * v if k == "l0.mix.dkv.norm" else v) for k, v in w.items()}
    assert "l3.mix.dkv" not in w and cases.logit_error(orc.forward(cfg, loud, toks), want)[20:].min() > 1e-3


@pytest.mark.parametrize("kind", ["attention", "latent_attention"])
def test_the_finder_finds(kind):
    cfg, w = cases.finder(kind, 200)
    toks = [t % cases.COMMON for t in cases.tokens(cfg, 190, seed=2)]
    toks[3], toks[-1] = cases.RARE, cases.ASK
    other = list(toks)
    other[3] = cases.COMMON
    assert cases.logit_error(orc.forward(cfg, w, toks)[-1:], orc.forward(cfg, w, other)[-1:])[0] > 5 * cases.TOLERANCE["bfloat16"]


# ---- configuration and layout -------------------------------------------------------------------------------------------

def test_configuration_reader():
    d, *_ = cases.MODELS["mixed"]
    cfg = lebelix.config_from_json(d, max_tokens=77)
    assert cfg.n_layer == 5 and cfg.max_tokens == 77 and cfg.layers[1].columns == 240 and cfg.layers[3].ff == 0 and cfg.layers[3].kv_from == 0
    assert (cfg.layers[1].softcap, cfg.layers[1].mask_size, cfg.layers[1].rot_dims, cfg.embed_scale, cfg.side_dim) == (9.0, 23, 20, 1.7, 20)

    def broken(layer, path, value):
        bad = json.loads(json.dumps(d))
        at = bad["layers"][layer]
        for p in path[:-1]:
            at = at[p]
        at[path[-1]] = value
        with pytest.raises(ValueError):
            lebelix.config_from_json(bad)

    broken(0, ("type",), "other")
    broken(0, ("mlp", "kind"), "experts")
    broken(0, ("mixer", "rot_dim"), 8)
    broken(1, ("mixer", "kv_heads"), 4)
    broken(1, ("mixer", "rot", "dims"), 50)
    for j in (1, 3, -1):
        broken(3, ("mixer", "kv_from"), j)
    broken(3, ("mixer", "kv_rank"), 55)


def test_packed_layers_hold_every_weight_once():
    """The stacked matrices of a layer multiply like the separate ones."""
    d, *ranks = cases.MODELS["mixed"]
    cfg, w = lebelix.config_from_json(d, dtype="float32"), cases.weights(d, *ranks)
    pk = hybrid.Packer(lambda n: w[n], cfg.weight_type)
    x = np.random.default_rng(0).standard_normal(cfg.width).astype(np.float32)
    xp = np.zeros(192, dtype=np.float32)
    xp[:cfg.width] = x
    for i, names in ((0, ("q", "dkv")), (1, ("q", "k", "v", "g")), (2, ("q", "k", "v", "b", "a1", "g1")), (3, ("q",))):
        scalars, arrays = lebelix._pack_layer(pk, cfg, i)
        y, row = arrays["w_in"] @ xp + arrays["b_in"], 0
        for n in names:
            m = w[f"l{i}.mix.{n}"]
            want = m @ x + (w[f"l{i}.mix.{n}.b"] if i == 1 and n != "g" else 0)
            assert row % 32 == 0 and np.allclose(y[row:row + len(m)], want, atol=1e-5)
            row += -(-len(m) // 32) * 32
        assert row == len(y)
        assert np.allclose(arrays["norm"][:cfg.width], 1 + w[f"l{i}.norm1"]) and ("norm2" in arrays) == (scalars["ff"] > 0)
        if i in (0, 3):
            uk, uv = w[f"l{i}.mix.uk"], w[f"l{i}.mix.uv"]
            at = -(-len(uk) // 32) * 32
            assert np.array_equal(arrays["w_latent"][:len(uk), :56], uk) and np.array_equal(arrays["w_latent"][at:at + len(uv), :56], uv)
        if i == 2:
            assert np.allclose(arrays["decay_rate"], np.exp(w["l2.mix.A_log"])) and arrays["conv"].shape == (2 * 3 * 40 + 6 * 24, 3)


def test_missing_or_misshapen_tensors_are_named():
    d, *ranks = cases.MODELS["odd"]
    cfg, w = lebelix.config_from_json(d), cases.weights(d, *ranks)
    w["l0.mix.k.conv"] = w["l0.mix.k.conv"][:-1]
    with pytest.raises(ValueError, match="l0.mix.k.conv"):
        lebelix._pack_layer(hybrid.Packer(lambda n: w[n], cfg.weight_type), cfg, 0)


def test_registry(tmp_path):
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Lebelix"}))
    assert models.architecture_of(str(tmp_path)) == "Lebelix" and "Lebelix" in models.ARCHITECTURES
