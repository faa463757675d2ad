"""CPU: the Nusilix oracle against closed forms, that the small test models react to every mechanism (so that a parity test on
them can fail), the safetensors container, the configuration reader and the registry."""
import json

import nusilix_cases as cases
import numpy as np
import pytest

from oracle import nusilix_oracle as orc
from skainet_amd import hybrid, models, nusilix
from skainet_amd.safetensors import SafetensorsReader, bf16_to_f32, f32_to_bf16, write_safetensors


def test_sinusoid_and_temperature_known_values():
    s = orc.sinusoid([0, 1, 5], 6)
    assert np.allclose(s[0], [0, 1, 0, 1, 0, 1])
    assert np.allclose(s[2, 2:4], [np.sin(5 * 10000 ** (-2 / 6)), np.cos(5 * 10000 ** (-2 / 6))])
    t = orc.query_temperature(np.arange(20), 0.5, 8)
    assert np.all(t[:7] == 1.0) and np.allclose(t[7:15], 1 + 0.5 * np.log(2)) and np.allclose(t[15:], 1 + 0.5 * np.log(3))
    assert np.allclose(orc.distance_slopes(8), 2.0 ** -np.arange(1, 9))


def test_grouped_norm_is_a_norm_per_part():
    x = np.array([[3.0, 4.0, 0.0, 10.0]])
    y = orc.grouped_rms_norm(x, np.array([1.0, 2.0, 3.0, 4.0]), 0.0, 2)
    assert np.allclose(y, [[3 / np.sqrt(12.5), 8 / np.sqrt(12.5), 0.0, 40 / np.sqrt(50)]])
    assert np.allclose(orc.grouped_rms_norm(x, np.ones(4), 1e-3, 1), orc.rms_norm(x, np.ones(4), 1e-3))


def test_xielu_limits():
    assert orc.xielu(np.array(0.0), 0.3, -0.2) == 0.0
    assert np.isclose(orc.xielu(np.array(2.0), 0.0, 1.0), np.log(2) * 4 + 1)
    z = -30.0
    assert np.isclose(orc.xielu(np.array(z), 0.0, 0.0), (0.5 + np.log(2)) * (-1 - z) + z / 2)


def test_attention_of_one_token_and_of_equal_scores():
    k = np.random.default_rng(0).standard_normal((5, 1, 4))
    out = orc.shared_kv_attention(np.zeros((5, 2, 4)), k, k, 1.0, np.zeros(2), 0)
    assert np.allclose(out[0, 0], k[0, 0]) and np.allclose(out[4, 1], k[:, 0].mean(axis=0))
    steep = orc.shared_kv_attention(np.zeros((5, 1, 4)), k, k, 1.0, np.array([1000.0]), 0)
    assert np.allclose(steep[4, 0], k[4, 0])  # the bias leaves the newest key only


def test_delta_rule_special_cases():
    rng = np.random.default_rng(1)
    r, k, v = (rng.standard_normal((6, 1, 3)) for _ in range(3))
    one, zero = np.ones((6, 1, 3)), np.zeros((6, 1, 3))
    o, _ = orc.generalized_delta_rule(r, k, v, one, zero)  # nothing forgotten or removed: linear attention
    want = [sum((r[t, 0] @ k[s, 0]) * v[s, 0] for s in range(t + 1)) for t in range(6)]
    assert np.allclose(o[:, 0], want)
    o, _ = orc.generalized_delta_rule(k, k, v, one, one)  # full removal along the key: the stored value is |k|^2 v
    assert np.allclose(o[:, 0], (k[:, 0] ** 2).sum(axis=1, keepdims=True) * v[:, 0], atol=1e-5)
    a = orc.generalized_delta_rule(r, k, v, 0.7 * one, 0.4 * one)
    first, state = orc.generalized_delta_rule(r[:2], k[:2], v[:2], 0.7 * one[:2], 0.4 * one[:2])
    rest, state = orc.generalized_delta_rule(r[2:], k[2:], v[2:], 0.7 * one[2:], 0.4 * one[2:], state)
    assert np.allclose(np.concatenate([first, rest]), a[0]) and np.allclose(state, a[1])


MUTATIONS = {
    "no distance bias": ("distance_slopes", lambda f: lambda heads: np.zeros(heads)),
    "slopes of the next head": ("distance_slopes", lambda f: lambda heads: np.roll(f(heads), 1)),
    "no temperature": ("query_temperature", lambda f: lambda p, coef, every: np.ones(len(p))),
    "positions from 1": ("sinusoid", lambda f: lambda p, width: f(np.asarray(p) + 1, width)),
    "norm in one group": ("grouped_rms_norm", lambda f: lambda x, w, eps, groups: f(x, w, eps, 1)),
    "no removal": ("unit_key", lambda f: lambda k: np.zeros_like(k)),
    "decay without the square root": ("delta_decay", lambda f: lambda z, w0: f(z, w0) ** np.exp(-0.5)),
    "activation without its linear part": ("xielu", lambda f: lambda z, p, q: f(z, p, q) - 0.5 * z),
}


@pytest.mark.parametrize("what", sorted(MUTATIONS))
def test_the_models_react_to_every_mechanism(what, monkeypatch):
    cfg, rank = cases.MODELS["mixed"]
    w = cases.weights(cfg, rank)
    toks = cases.tokens(cfg, 40)
    want = orc.forward(cfg, w, toks)
    name, mutate = MUTATIONS[what]
    monkeypatch.setattr(orc, name, mutate(getattr(orc, name)))
    err = cases.logit_error(orc.forward(cfg, w, toks), want)
    assert np.median(err[8:]) > 1.5 * cases.TOLERANCE["bfloat16"], err
    assert err[8:].min() > 20 * cases.TOLERANCE["float32"]


def test_a_temperature_one_token_late_shows_where_it_steps(monkeypatch):
    cfg, rank = cases.MODELS["mixed"]
    w, toks = cases.weights(cfg, rank), cases.tokens(cfg, 40)
    want, f = orc.forward(cfg, w, toks), orc.query_temperature
    monkeypatch.setattr(orc, "query_temperature", lambda p, coef, every: f(np.asarray(p) - 1, coef, every))
    err = cases.logit_error(orc.forward(cfg, w, toks), want)
    assert err[[6, 13, 20, 27]].min() > 100 * cases.TOLERANCE["float32"]


def test_values_are_the_keys_before_their_norm():
    cfg, rank = cases.MODELS["attention_64"]
    w = cases.weights(cfg, rank)
    toks = cases.tokens(cfg, 20)
    want = orc.forward(cfg, w, toks)
    w2 = {k: (2.0 * v if k.endswith("k.norm") else v) for k, v in w.items()}
    assert cases.logit_error(orc.forward(cfg, w2, toks), want)[0] < 1e-12  # one key: its norm's weights do not matter
    assert cases.logit_error(orc.forward(cfg, w2, toks), want)[5:].min() > 1e-3


# ---- files and configuration -------------------------------------------------------------------------------------------

def test_safetensors_round_trip(tmp_path):
    a = np.random.default_rng(0).standard_normal((3, 5)).astype(np.float32)
    table = np.arange(4, dtype=np.int32)
    write_safetensors(tmp_path / "m.safetensors", {"a": a, "table": table})
    r = SafetensorsReader(tmp_path / "m.safetensors")
    assert r.names() == ["a", "table"] and r.shape("a") == (3, 5) and r.dtype("a") == "BF16" and "b" not in r
    assert np.array_equal(r.raw("a"), f32_to_bf16(a)) and np.array_equal(r.f32("a"), bf16_to_f32(f32_to_bf16(a)))
    assert np.array_equal(r.raw("table"), table) and r.raw("table").dtype == np.int32
    with pytest.raises(ValueError, match="no tensor"):
        r.raw("b")
    r.close()
    (tmp_path / "bad").write_bytes(b"\xff" * 64)
    with pytest.raises(ValueError):
        SafetensorsReader(tmp_path / "bad")


def test_bf16_rounding_is_to_nearest_even():
    x = np.array([1.0, 1.0 + 2.0 ** -8, 1.0 + 3 * 2.0 ** -8, -2.0 - 2.0 ** -6], dtype=np.float32)
    assert bf16_to_f32(f32_to_bf16(x)).tolist() == [1.0, 1.0, 1.0 + 2.0 ** -6, -2.0 - 2.0 ** -6]


def test_configuration_reader():
    cfg_dict, _ = cases.MODELS["mixed"]
    cfg = nusilix.config_from_json(cfg_dict, max_tokens=77)
    assert cfg.n_layer == 4 and cfg.max_tokens == 77 and cfg.layers[1].columns == 120 and cfg.layers[3].ff == 0
    assert (cfg.layers[0].temp_coef, cfg.layers[0].temp_every) == (0.4, 7.0)
    for path, value in ((("type",), "other"), (("mixer", "vdim"), 5), (("mlp", "kind"), "experts")):
        bad = json.loads(json.dumps(cfg_dict))
        at = bad["layers"][0]
        for p in path[:-1]:
            at = at[p]
        at[path[-1]] = value
        with pytest.raises(ValueError):
            nusilix.config_from_json(bad)


def test_packed_layer_holds_every_weight_once():
    """The stacked and joined matrices of a layer multiply like the separate ones."""
    cfg_dict, rank = cases.MODELS["mixed"]
    cfg, w = nusilix.config_from_json(cfg_dict, dtype="float32"), cases.weights(cfg_dict, rank)
    pk = hybrid.Packer(lambda n: w[n], cfg.weight_type)
    x = np.random.default_rng(0).standard_normal(cfg.width).astype(np.float32)
    xp = np.zeros(192, dtype=np.float32)
    xp[:cfg.width] = x
    for i, names in ((0, ("mix.q", "mix.k", "mlp.up")), (1, ("mix.r", "mix.k", "mix.v", "mix.g", "mix.a", "mix.w1", "mlp.up"))):
        _, arrays = nusilix._pack_layer(pk, cfg, i)
        y, row = arrays["w_in"] @ xp + arrays["b_in"], 0
        for n in names:
            m = w[f"l{i}.{n}"]
            want = m @ x + w.get(f"l{i}.{n}.b", np.zeros(len(m), dtype=np.float32))
            assert row % 32 == 0 and np.allclose(y[row:row + len(m)], want, atol=1e-5)
            row += -(-len(m) // 32) * 32
        assert row == len(y)
        o, down = w[f"l{i}.mix.o"], w[f"l{i}.mlp.down"]
        off = -(-o.shape[1] // 64) * 64
        assert np.array_equal(arrays["w_out"][:cfg.width, :o.shape[1]], o) and np.array_equal(arrays["w_out"][:cfg.width, off:off + down.shape[1]], down)
        assert np.count_nonzero(arrays["w_out"]) == np.count_nonzero(o) + np.count_nonzero(down)


def test_missing_or_misshapen_tensors_are_named():
    cfg_dict, rank = cases.MODELS["odd"]
    cfg, w = nusilix.config_from_json(cfg_dict), cases.weights(cfg_dict, rank)
    w["l1.mix.q"] = w["l1.mix.q"][:-1]
    with pytest.raises(ValueError, match="l1.mix.q"):
        nusilix._pack_layer(hybrid.Packer(lambda n: w[n], cfg.weight_type), cfg, 1)


def test_registry(tmp_path):
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Nusilix"}))
    assert models.architecture_of(str(tmp_path)) == "Nusilix"
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Unheard"}))
    with pytest.raises(ValueError, match="Unheard"):
        models.load_model(None, str(tmp_path))
    assert "llama" in models.ARCHITECTURES
