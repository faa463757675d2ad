"""GPU: the mechanisms of the Nusilix decoder one at a time against the slow oracle -- norm in groups, xIELU, attention over a shared
key/value cache (prompts, portions, single tokens, pages freed and used again), the generalized delta rule with its state."""
import numpy as np
import pytest

from oracle import nusilix_oracle as orc
from skainet_amd import runtime

pytestmark = pytest.mark.gpu


def rel(got, want):
    return np.abs(np.asarray(got, dtype=np.float64) - want).max() / np.abs(want).max()


# ---- norm and activation -----------------------------------------------------------------------------------------------

@pytest.mark.parametrize("rows,n,groups", [(1, 64, 1), (3, 45, 9), (5, 200, 2), (2, 4096, 4), (4, 1000, 8), (7, 30, 30), (2, 257, 1)])
def test_grouped_norm(hip, rows, n, groups):
    rng = np.random.default_rng(n + groups)
    x = (rng.standard_normal((rows, n)) * np.exp(rng.standard_normal((rows, 1)))).astype(np.float32)
    x[:, :n // groups] *= 40.0  # (one loud part: a norm over the whole row would show)
    w = (1 + 0.3 * rng.standard_normal(n)).astype(np.float32)
    y = hip.alloc(x.nbytes)
    hip.rmsnorm_grouped(hip.to_device(x), hip.to_device(w), rows, n, groups, 1e-5, y)
    want = orc.grouped_rms_norm(x.astype(np.float64), w.astype(np.float64), 1e-5, groups)
    assert np.abs(y.download(np.float32, x.size).reshape(x.shape) - want).max() < 2e-6 * np.abs(want).max()


def test_grouped_norm_refuses_unequal_parts(hip):
    b = hip.alloc(4 * 100)
    with pytest.raises(runtime.SknError):
        hip.rmsnorm_grouped(b, b, 1, 100, 3, 1e-5, b)


def test_xielu(hip):
    z = np.concatenate([np.linspace(-40, 20, 4001), np.geomspace(1e-8, 1, 200), -np.geomspace(1e-8, 1, 200), [0.0, -0.35, -0.3500001]]).astype(np.float32)
    p, q = 0.8, -0.6
    out = hip.alloc(z.nbytes)
    hip.xielu(hip.to_device(z), z.size, float(orc.softplus(p)), 0.5 + float(orc.softplus(q)), out)
    want = orc.xielu(z.astype(np.float64), p, q)
    got = out.download(np.float32, z.size)
    assert np.all(np.abs(got - want) <= 1e-6 * (np.abs(want) + np.abs(z)) + 1e-12)


# ---- attention ---------------------------------------------------------------------------------------------------------

def attn_case(heads, kv_heads, dim, n, seed, coef=0.3, every=11, scale=None):
    rng = np.random.default_rng(seed)
    q = rng.standard_normal((n, heads * dim)).astype(np.float32) * 1.7
    k = rng.standard_normal((n, kv_heads * dim)).astype(np.float32) * 0.6
    p = {"n_head": heads, "scale": dim ** -0.5 if scale is None else scale, "temp_coef": coef, "temp_every": every, "eps": 1e-5,
         "q_norm": (1 + 0.3 * rng.standard_normal(heads * dim)).astype(np.float32), "k_norm": (1 + 0.3 * rng.standard_normal(kv_heads * dim)).astype(np.float32)}
    return q, k, p


def attn_oracle(q, k, p, heads, kv_heads, dim):
    n = len(q)
    q, k = q.astype(np.float64), k.astype(np.float64)
    qn = orc.rms_norm(q, p["q_norm"].astype(np.float64), p["eps"])
    if p["temp_coef"]:
        qn = qn * orc.query_temperature(np.arange(n), p["temp_coef"], p["temp_every"])[:, None]
    kn = orc.rms_norm(k, p["k_norm"].astype(np.float64), p["eps"])
    o = orc.shared_kv_attention(qn.reshape(n, heads, dim), kn.reshape(n, kv_heads, dim), k.reshape(n, kv_heads, dim), p["scale"], orc.distance_slopes(heads), 0)
    return o.reshape(n, heads * dim)


TOL = {runtime.F16: 4e-3, runtime.F32: 3e-6}
SHAPES = [(4, 4, 64), (6, 2, 64), (8, 1, 128), (3, 3, 20), (4, 2, 96), (2, 1, 256), (5, 5, 130)]


@pytest.mark.parametrize("elem", [runtime.F16, runtime.F32])
@pytest.mark.parametrize("heads,kv_heads,dim", SHAPES)
def test_shared_attention_in_one_go_in_portions_and_token_by_token(hip, heads, kv_heads, dim, elem):
    n = 150
    q, k, p = attn_case(heads, kv_heads, dim, n, seed=dim + heads)
    want = attn_oracle(q, k, p, heads, kv_heads, dim)
    kv = runtime.SharedKVCache(hip, 1, kv_heads, dim, 16, 192, elem)
    results = {}
    for name, cuts in (("whole", [n]), ("portions", [2, 3, 16, 31, 33, 2, 64]), ("tokens", [1] * n)):
        kv.reset()
        at, out = 0, []
        for c in cuts:
            c = min(c, n - at)
            if c:
                out.append(kv.attend(0, p, q[at:at + c], k[at:at + c]))
                at += c
        assert at >= n - 1 and kv.length(0) == at
        results[name] = np.concatenate(out)
        assert rel(results[name], want[:at]) < TOL[elem], name
    kv.free()


@pytest.mark.parametrize("elem", [runtime.F16, runtime.F32])
@pytest.mark.parametrize("far", [0, 1, 15, 16, 17, 31, 32, 63, 64, 127, 128, 254, 255, 256])
def test_one_far_key_stands_out(hip, elem, far):
    """Query 299 matches one key far away so well that it outweighs its distance: at page borders, tile borders, the first tokens."""
    heads, kv_heads, dim, n = 6, 2, 56, 300
    q, k, p = attn_case(heads, kv_heads, dim, n, seed=5, coef=0.0, scale=1.0)
    p["q_norm"][:], p["k_norm"][:] = 1.0, 1.0
    qh = q[299].reshape(heads, dim)
    k[far] = np.concatenate([qh[2], qh[5]])  # (head 2 reads cached head 0, head 5 cached head 1)
    want = attn_oracle(q, k, p, heads, kv_heads, dim)
    without = k.copy()
    without[far] = -k[far]
    gone = attn_oracle(q, without, p, heads, kv_heads, dim)
    assert np.abs(want[299] - gone[299]).max() > 0.5 * np.abs(want[299]).max()  # (losing that key would show)
    kv = runtime.SharedKVCache(hip, 1, kv_heads, dim, 16, 320, elem)
    head = kv.attend(0, p, q[:299], k[:299])
    last = kv.attend(0, p, q[299:], k[299:])
    assert rel(head, want[:299]) < TOL[elem] and rel(last, want[299:]) < TOL[elem]
    kv.reset()
    assert rel(kv.attend(0, p, q, k), want) < TOL[elem]
    kv.free()


def test_pages_that_are_freed_and_used_again_by_other_sequences(hip):
    heads, kv_heads, dim = 4, 2, 48
    kv = runtime.SharedKVCache(hip, 3, kv_heads, dim, 8, 64)
    cases = {s: attn_case(heads, kv_heads, dim, n, seed=40 + s) for s, n in ((0, 50), (1, 17), (2, 33))}
    for turn in range(3):
        order = [0, 1, 2] if turn % 2 == 0 else [2, 0, 1]
        for s in order:  # (three sequences grow in turns, then one is dropped and starts again)
            q, k, p = cases[s]
            kv.reset(s)
            half = len(q) // 2
            a = kv.attend(s, p, q[:half], k[:half])
            other = order[(order.index(s) + 1) % 3]
            if kv.length(other):
                kv.reset(other)
            b = kv.attend(s, p, q[half:], k[half:])
            assert rel(np.concatenate([a, b]), attn_oracle(q, k, p, heads, kv_heads, dim)) < TOL[runtime.F16], (turn, s)
    kv.free()


def test_shared_cache_errors(hip):
    kv = runtime.SharedKVCache(hip, 1, 2, 32, 8, 16)
    q, k, p = attn_case(4, 2, 32, 17, seed=1)
    with pytest.raises(runtime.SknError) as e:
        kv.attend(0, p, q, k)
    assert e.value.code == runtime.ERR_POOL
    with pytest.raises(runtime.SknError):
        kv.attend(1, p, q[:3], k[:3])
    buf = hip.alloc(4096)
    assert hip.lib.skn_attn_decode(hip.handle, kv.handle, buf.ptr, None, 1.0, buf.ptr) == runtime.ERR_STATE
    assert hip.lib.skn_kv_append_run(hip.handle, kv.handle, 0, buf.ptr, buf.ptr, 1) == runtime.ERR_STATE
    assert hip.lib.skn_attn_prefill(hip.handle, kv.handle, 0, buf.ptr, 1, 1.0, buf.ptr) in (runtime.ERR_STATE, runtime.ERR_RANGE)
    kv.free()
    with pytest.raises(runtime.SknError):
        runtime.SharedKVCache(hip, 1, 2, 257, 8, 16)
    with pytest.raises(runtime.SknError):
        runtime.SharedKVCache(hip, 1, 2, 64, 8, 16, elem_type=runtime.Q4_K)


# ---- generalized delta rule --------------------------------------------------------------------------------------------

def delta_case(heads, dim, n, seed, slow=False):
    rng = np.random.default_rng(seed)
    r, k, v = (rng.standard_normal((n, heads * dim)).astype(np.float32) for _ in range(3))
    z = rng.standard_normal((n, heads * dim)) * (1 if slow else 3) - (9 if slow else 0)
    decay = orc.delta_decay(z, 0.0).astype(np.float32)
    rate = orc.sigmoid(2 * rng.standard_normal((n, heads * dim))).astype(np.float32)
    return r * dim ** -0.5, k * dim ** -0.25, v, decay, rate


def delta_oracle(c, heads, dim):
    o, _ = orc.generalized_delta_rule(*(a.astype(np.float64).reshape(len(a), heads, dim) for a in c))
    return o.reshape(len(o), heads * dim)


@pytest.mark.parametrize("heads,dim", [(1, 1), (2, 5), (3, 16), (2, 32), (3, 33), (2, 64), (1, 100), (2, 128), (1, 129), (1, 256)])
def test_delta_rule_in_one_go_in_portions_and_token_by_token(hip, heads, dim):
    n = 70
    c = delta_case(heads, dim, n, seed=dim)
    want = delta_oracle(c, heads, dim)
    st = runtime.RecurrentState(hip, 1, heads, dim)
    for cuts in ([n], [2, 3, 16, 15, 17, 1, 16], [1] * 20 + [50]):
        st.reset()
        at, out = 0, []
        for m in cuts:
            out.append(st.advance(0, *(a[at:at + m] for a in c)))
            at += m
        assert at == n
        assert rel(np.concatenate(out), want) < 1e-5, cuts
    st.free()


def test_delta_rule_remembers_over_a_long_sequence(hip):
    """Decays near one: the first token's value is still in the state a thousand tokens later."""
    heads, dim, n = 2, 24, 1000
    c = delta_case(heads, dim, n, seed=3, slow=True)
    rate = np.zeros_like(c[4])
    c = (*c[:4], rate)
    want = delta_oracle(c, heads, dim)
    v2 = c[2].copy()
    v2[0] += 5
    assert rel(delta_oracle((c[0], c[1], v2, c[3], rate), heads, dim)[-1], want[-1]) > 1e-3
    st = runtime.RecurrentState(hip, 1, heads, dim)
    assert rel(st.advance(0, *c), want) < 2e-5
    st.free()


def test_states_of_several_sequences_stay_apart_and_reset(hip):
    heads, dim = 2, 40
    a, b = delta_case(heads, dim, 20, seed=1), delta_case(heads, dim, 31, seed=2)
    st = runtime.RecurrentState(hip, 3, heads, dim)
    for _ in range(2):
        x0 = st.advance(0, *(z[:9] for z in a))
        y0 = st.advance(2, *(z[:11] for z in b))
        x1 = st.advance(0, *(z[9:] for z in a))
        y1 = st.advance(2, *(z[11:] for z in b))
        assert rel(np.concatenate([x0, x1]), delta_oracle(a, heads, dim)) < 1e-5
        assert rel(np.concatenate([y0, y1]), delta_oracle(b, heads, dim)) < 1e-5
        st.reset(0)
        assert rel(st.advance(0, *a), delta_oracle(a, heads, dim)) < 1e-5
        st.reset()
    st.free()


def test_many_heads(hip):
    heads, dim, n = 80, 64, 33
    c = delta_case(heads, dim, n, seed=9)
    st = runtime.RecurrentState(hip, 1, heads, dim)
    assert rel(st.advance(0, *c), delta_oracle(c, heads, dim)) < 1e-5
    st.free()
