"""GPU: Nusilix models end to end against the slow oracle -- prompts, token by token, portions of prompts, requests one after the
other, far keys in decoding, long greedy decoding, and the framework's own entry points (registry, generation, trace replay)."""
import json
import os
import subprocess

import nusilix_cases as cases
import numpy as np
import pytest

from oracle import nusilix_oracle as orc
from skainet_amd import generate, models, nusilix, runtime
from skainet_amd.safetensors import write_safetensors
from skainet_amd.trace import Replay

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = ["float32", "bfloat16"]


def run(model, toks, cuts, want=None):
    """Feeds the tokens in portions; logits of every token (or of the places in `want`)."""
    model.reset()
    at, out = 0, []
    for c in cuts:
        c = min(c, len(toks) - at)
        if c:
            places = [p - at for p in (range(len(toks)) if want is None else want) if at <= p < at + c]
            out.append(model.extend(toks[at:at + c], places))
            at += c
    assert at == len(toks)
    return np.concatenate(out)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(cases.MODELS))
def test_prompts_portions_and_single_tokens_match_the_oracle(hip, name, dtype):
    cfg, rank = cases.MODELS[name]
    w = cases.weights(cfg, rank, seed=len(name))
    toks = cases.tokens(cfg, 100)
    want = orc.forward(cfg, w, toks)
    m = cases.device_model(hip, cfg, w, dtype)
    for cuts in ([100], [1] * 100, [2, 3, 5, 16, 17, 31, 2, 24], [60] + [1] * 40):
        cases.check(run(m, toks, cuts), want, dtype, cuts[:4])
    m.free()


@pytest.mark.parametrize("dtype", DTYPES)
def test_logits_do_not_depend_on_the_cut(hip, dtype):
    cfg, rank = cases.MODELS["mixed"]
    w = cases.weights(cfg, rank)
    toks = cases.tokens(cfg, 200, seed=4)
    m = cases.device_model(hip, cfg, w, dtype)
    whole = run(m, toks, [200])
    assert np.array_equal(whole, run(m, toks, [200]))  # (and nothing is left over from the run before)
    for size in (2, 3, 7, 16, 50, 64, 127):
        err = cases.logit_error(run(m, toks, [size] * 100), whole)
        assert err.max() < cases.TOLERANCE[dtype] / (1 if dtype == "float32" else 4), size
    m.free()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("tile", [1, 2, 3, 4, 5])
def test_every_tile_of_the_gemm(hip, tile, dtype):
    cfg, rank = cases.MODELS["mixed"]
    w = cases.weights(cfg, rank)
    toks = cases.tokens(cfg, 300, seed=5)
    want = orc.forward(cfg, w, toks)
    m = cases.device_model(hip, cfg, w, dtype)
    hip.set_option("dense.tile", tile)
    try:
        err = cases.logit_error(run(m, toks, [300]), want)
    finally:
        hip.set_option("dense.tile", 0)
    assert err.max() < cases.TOLERANCE[dtype]
    m.free()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv_heads,dim", [(8, 2, 64), (8, 8, 32), (4, 1, 128), (3, 1, 200)])
def test_a_far_key_is_found_in_prompts_and_in_decoding(hip, heads, kv_heads, dim, dtype):
    cfg, w = cases.finder(heads, kv_heads, dim)
    n = 300
    toks = [t % cases.COMMON for t in cases.tokens(cfg, n, seed=2)]
    m = cases.device_model(hip, cfg, w, dtype, page_tokens=16)
    for far in (0, 1, 15, 16, 31, 32, 127, 128, 255, 256, 270):
        t = list(toks)
        t[far], t[-1] = cases.RARE, cases.ASK
        want = orc.forward(cfg, w, t)
        other = list(t)
        other[far] = cases.COMMON
        assert cases.logit_error(orc.forward(cfg, w, other)[-1:], want[-1:])[0] > 5 * cases.TOLERANCE[dtype]
        for cuts in ([n], [n - 1, 1], [far + 1, n - far - 1], [n - 40] + [1] * 40):
            got = run(m, t, cuts, want=[n - 1])
            assert cases.logit_error(got, want[-1:])[0] < cases.TOLERANCE[dtype], (far, cuts[:2])
    m.free()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv_heads,dim", [(6, 2, 48), (5, 5, 9), (4, 1, 100), (2, 2, 200), (24, 2, 64)])
def test_decoding_over_contexts_that_are_split(hip, heads, kv_heads, dim, dtype):
    """Contexts past 512 and 1024 tokens: several workgroups share a head's keys and the output product's staging merges them."""
    cfg, w = cases.finder(heads, kv_heads, dim, match=22.0)
    n = 1100
    toks = [t % cases.COMMON for t in cases.tokens(cfg, n, seed=7)]
    m = cases.device_model(hip, cfg, w, dtype, max_tokens=1200, page_tokens=64)
    for far in (0, 63, 64, 511, 512, 1023, 1024):
        t = list(toks)
        t[far], t[-1] = cases.RARE, cases.ASK
        want = orc.forward(cfg, w, t)
        other = list(t)
        other[far] = cases.COMMON
        assert cases.logit_error(orc.forward(cfg, w, other)[-1:], want[-1:])[0] > 5 * cases.TOLERANCE[dtype]
        got = run(m, t, [n - 12] + [1] * 12, want=range(n - 14, n))
        cases.check(got, want[n - 14:], dtype, far)
    m.free()


def test_requests_one_after_the_other_use_pages_and_states_again(hip):
    cfg, rank = cases.MODELS["mixed"]
    w = cases.weights(cfg, rank)
    m = cases.device_model(hip, cfg, w, max_tokens=128, page_tokens=8)
    for seed, n in ((1, 100), (2, 5), (3, 128), (4, 1), (5, 77), (6, 2)):
        toks = cases.tokens(cfg, n, seed=seed)
        cut = max(1, n - 6)
        assert cases.logit_error(run(m, toks, [cut] + [1] * 6), orc.forward(cfg, w, toks)).max() < cases.TOLERANCE["float32"], n
    m.free()


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_greedy_decoding_follows_the_oracle(hip, dtype):
    """Four hundred greedy tokens: every choice is the oracle's best (or as good as its best, within the tolerance)."""
    cfg, rank = cases.MODELS["deep"]
    w = cases.weights(cfg, rank)
    m = cases.device_model(hip, cfg, w, dtype, max_tokens=448)
    prompt = cases.tokens(cfg, 40, seed=8)
    out = m.generate(prompt, 401)
    assert len(out) == 401
    want = orc.forward(cfg, w, prompt + out[:-1])
    rows = want[len(prompt) - 1:]
    room = 6 * cases.TOLERANCE[dtype] * np.sqrt(((want - want.mean(axis=1, keepdims=True)) ** 2).mean())
    best = rows.max(axis=1)
    chosen = rows[np.arange(401), out]
    assert np.all(best - chosen <= room)
    assert cases.logit_error(m.logits()[None], rows[-1:])[0] < cases.TOLERANCE[dtype]
    m.free()


def test_captured_steps_equal_eager_ones_on_every_replay(hip):
    cfg, rank = cases.MODELS["mixed"]
    w = cases.weights(cfg, rank)
    m = cases.device_model(hip, cfg, w, "bfloat16")
    toks = cases.tokens(cfg, 60, seed=3)
    res = {}
    for graph in (0, 1):
        hip.set_option("llama.graph", graph)
        if graph and hip.stat("profiler.attached"):
            pytest.skip("a profiler is attached: steps are not captured")
        m.reset()
        rows = [m.extend(toks[:20], [19])]
        for t in toks[20:]:
            rows.append(m.extend([t], [0]))
            hip.sync()
        res[graph] = np.concatenate(rows)
    assert np.array_equal(res[0], res[1])
    m.free()


def test_decode_in_one_call_equals_many_calls(hip):
    cfg, rank = cases.MODELS["mixed"]
    m = cases.device_model(hip, cfg, cases.weights(cfg, rank), "bfloat16", max_tokens=512)
    prompt = cases.tokens(cfg, 33, seed=6)
    a = m.generate(prompt, 150)  # (past 128 tokens, where the step is captured again)
    m.reset()
    b = [m.prefill(prompt)]
    while len(b) < 150:
        b += m.decode(b[-1], min(7, 150 - len(b)))
    assert a == b
    m.free()


def test_a_long_prompt_runs_in_slices(hip):
    """More tokens than one slice of the prompt buffers holds (8192)."""
    cfg = cases.model([cases.attention(4, 1, 16, ff=0), cases.delta(2, 8, ff=0)], width=32, vocab=40, groups=2)
    w = cases.weights(cfg, 4)
    toks = cases.tokens(cfg, 8203, seed=1)
    m = cases.device_model(hip, cfg, w, max_tokens=8300, page_tokens=256)
    want = [5, 8190, 8191, 8192, 8193, 8202]
    whole = run(m, toks, [8203], want=want)
    assert cases.logit_error(run(m, toks, [8191, 5, 7], want=want), whole).max() < cases.TOLERANCE["float32"]
    assert cases.logit_error(run(m, toks, [4096, 4100, 1, 1, 5], want=want), whole).max() < cases.TOLERANCE["float32"]
    m.free()


def test_wanted_places_in_any_order_and_none(hip):
    cfg, rank = cases.MODELS["odd"]
    m = cases.device_model(hip, cfg, cases.weights(cfg, rank))
    toks = cases.tokens(cfg, 20)
    full = run(m, toks, [20])
    m.reset()
    assert m.extend(toks[:9], []).shape == (0, cfg["vocab"])
    assert cases.logit_error(m.extend(toks[9:], [7, 0, 10]), full[[16, 9, 19]]).max() < cases.TOLERANCE["float32"]
    m.free()


def test_errors_are_reported(hip):
    cfg, rank = cases.MODELS["odd"]
    m = cases.device_model(hip, cfg, cases.weights(cfg, rank), max_tokens=10)
    with pytest.raises(runtime.SknError) as e:
        m.extend([0] * 11)
    assert e.value.code == runtime.ERR_POOL
    with pytest.raises(runtime.SknError) as e:
        m.extend([cfg["vocab"]])
    assert e.value.code == runtime.ERR_RANGE
    m.extend([1] * 9)
    with pytest.raises(runtime.SknError):
        m.decode(1, 2)
    assert len(m.decode(1, 1)) == 1
    m.free()


@pytest.fixture
def model_folder(tmp_path):
    cfg, rank = cases.MODELS["mixed"]
    w = cases.weights(cfg, rank)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    write_safetensors(tmp_path / "model.safetensors", w)
    return tmp_path, cfg, w


@pytest.mark.parametrize("dtype", DTYPES)
def test_registry_generation_and_command_line(hip, model_folder, dtype, capsys):
    path, cfg, w = model_folder
    m = models.load_model(hip, str(path), dtype=dtype, max_tokens=64)
    assert isinstance(m, nusilix.NusilixModel)
    prompt = cases.tokens(cfg, 12, seed=9)
    out = m.generate(prompt, 20)
    assert out == m.generate(prompt, 20)
    m.free()
    direct = cases.device_model(hip, cfg, w, dtype, page_tokens=256)
    assert direct.generate(prompt, 20) == out
    direct.free()
    assert generate.main(["--model", str(path), "--prompt", ",".join(map(str, prompt)), "--tokens", "20", "--dtype", dtype]) == 0
    assert [int(t) for t in capsys.readouterr().out.split(",")] == out


def test_trace_replay(hip, model_folder):
    path, cfg, w = model_folder
    m = models.load_model(hip, str(path), dtype="float32", max_tokens=64)
    r = Replay(m)
    a, b = cases.tokens(cfg, 30, seed=1), cases.tokens(cfg, 9, seed=2)
    wa, wb = orc.forward(cfg, w, a), orc.forward(cfg, w, b)
    tol = cases.TOLERANCE["float32"]
    got = r.step([{"id": "a", "tokens": a[:13], "want": [12, 3]}], [])
    assert cases.logit_error(got, wa[[12, 3]]).max() < tol
    assert r.step([{"id": "a", "tokens": a[13:15], "want": []}], []).shape == (0, cfg["vocab"])
    with pytest.raises(ValueError, match="one sequence"):
        r.step([{"id": "b", "tokens": b, "want": []}], [])
    assert cases.logit_error(r.step([{"id": "a", "tokens": a[15:16], "want": [0]}], []), wa[[15]]).max() < tol
    assert cases.logit_error(r.step([{"id": "a", "tokens": a[16:], "want": [13]}], ["a"]), wa[[29]]).max() < tol
    assert cases.logit_error(r.step([{"id": "b", "tokens": b, "want": list(range(9))}], ["b"]), wb).max() < tol
    m.free()


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_program(model_folder, dtype):
    path, cfg, w = model_folder
    a, b = cases.tokens(cfg, 25, seed=3), cases.tokens(cfg, 6, seed=4)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:20], "want": [4, 19]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[20:22], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[22:23], "want": [0]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "b", "tokens": b, "want": [5]}], "end": ["b"]}]
    out = path / "out"
    out.mkdir()
    p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(path), "--dtype", dtype, "--out", str(out), "--max-tokens", "32"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=100)
    assert p.returncode == 0, p.stderr
    assert [line for line in p.stdout.splitlines() if line.startswith("done")] == [f"done {i}" for i in range(4)]
    assert sorted(os.listdir(out)) == ["0.f32", "2.f32", "3.f32"]
    wa, wb = orc.forward(cfg, w, a), orc.forward(cfg, w, b)
    for step, want in ((0, wa[[4, 19]]), (2, wa[[22]]), (3, wb[[5]])):
        got = np.fromfile(out / f"{step}.f32", dtype="<f4").reshape(-1, cfg["vocab"])
        assert cases.logit_error(got, want).max() < cases.TOLERANCE[dtype]
