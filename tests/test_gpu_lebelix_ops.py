"""GPU: the mechanisms of the Lebelix decoder one at a time against the slow oracle -- the activation, attention over ranges of the cache,
attention over latents (prompts, portions, single tokens, pages freed and used again), the gated delta rule with its convolutions."""
import numpy as np
import pytest

from oracle import lebelix_oracle as orc
from skainet_amd import runtime
from skainet_amd.hybrid import Packer
from skainet_amd.safetensors import bf16_to_f32, f32_to_bf16

pytestmark = pytest.mark.gpu
F16, F32 = runtime.F16, runtime.F32
TOL = {F16: 5e-3, F32: 4e-6}


def rel(got, want):
    return np.abs(np.asarray(got, dtype=np.float64) - want).max() / np.abs(want).max()


def in_portions(n, cuts, feed):
    at, out = 0, []
    for c in cuts:
        c = min(c, n - at)
        if c:
            out.append(feed(at, at + c))
            at += c
    assert at == n
    return np.concatenate(out)


def test_gelu(hip):
    z = np.concatenate([np.linspace(-30, 30, 4001), np.geomspace(1e-8, 1, 200), -np.geomspace(1e-8, 1, 200), [0.0]]).astype(np.float32)
    out = hip.alloc(z.nbytes)
    hip.gelu(hip.to_device(z), z.size, out)
    want = orc.gelu_tanh(z.astype(np.float64))
    assert np.all(np.abs(out.download(np.float32, z.size) - want) <= 2e-6 * np.abs(z) * (np.abs(want) > 1e-3) + 1e-6 * np.abs(z) + 1e-12)


# ---- attention over a range ------------------------------------------------------------------------------------------------

def ranged_case(heads, kv_heads, dim, vdim, n, seed, mask=None, rot=0, softcap=0.0, sink=0, norm=True, scale=None):
    rng = np.random.default_rng(seed)
    q, k, v = (rng.standard_normal((n, c)).astype(np.float32) for c in (heads * dim, kv_heads * dim, kv_heads * vdim))
    gate = orc.sigmoid(rng.standard_normal((n, heads * vdim))).astype(np.float32)
    p = {"n_head": heads, "scale": 2 * dim ** -0.5 if scale is None else scale, "eps": 1e-5, "mask": mask, "softcap": softcap, "sink": sink, "rot_dims": rot,
         "rot_base": 500.0}
    if norm:
        p["q_norm"], p["k_norm"] = ((1 + 0.3 * rng.standard_normal(dim)).astype(np.float32) for _ in range(2))
    return q, k, v, gate, p


def mask_of(p, n):
    kind, size = p["mask"] or (None, 0)
    return {"window": orc.window_mask, "chunk": orc.chunk_mask, None: lambda n, _: np.tril(np.ones((n, n), bool))}[kind](n, size)


def ranged_oracle(q, k, v, gate, p, kv_heads, dim, vdim):
    n, heads = len(q), p["n_head"]
    q, k, v = (a.astype(np.float64).reshape(n, -1, d) for a, d in ((q, dim), (k, dim), (v, vdim)))
    if "q_norm" in p:
        q, k = orc.plain_norm(q, p["q_norm"].astype(np.float64), p["eps"]), orc.plain_norm(k, p["k_norm"].astype(np.float64), p["eps"])
    q, k = (orc.rotate_half(a, np.arange(n), p["rot_base"], p["rot_dims"]) for a in (q, k))
    of = np.arange(heads) // (heads // kv_heads)
    s = np.einsum("thd,shd->hts", q, k[:, of]) * p["scale"]
    if p["softcap"]:
        s = orc.soft_cap(s, p["softcap"])
    w = (orc.sink_softmax if p["sink"] else orc.softmax)(s, mask_of(p, n))
    o = np.einsum("hts,shv->thv", w, v[:, of]).reshape(n, -1)
    return o if gate is None else o * gate


SHAPES = [(4, 4, 64, 64), (6, 2, 40, 64), (8, 1, 128, 128), (3, 3, 20, 7), (4, 2, 96, 72), (2, 1, 256, 256), (5, 5, 130, 12), (1, 1, 2, 200)]
FORMS = {"plain": {}, "all": dict(mask=("chunk", 37), softcap=4.0, sink=1), "window": dict(mask=("window", 21), sink=1), "one": dict(mask=("window", 1), softcap=2.0)}


@pytest.mark.parametrize("elem", [F16, F32])
@pytest.mark.parametrize("form", sorted(FORMS))
@pytest.mark.parametrize("heads,kv_heads,dim,vdim", SHAPES)
def test_ranged_attention_in_one_go_in_portions_and_token_by_token(hip, heads, kv_heads, dim, vdim, form, elem):
    n = 130
    rot = {"plain": 0, "all": dim // 2 // 2 * 2, "window": dim // 2 * 2, "one": 2}[form]
    q, k, v, gate, p = ranged_case(heads, kv_heads, dim, vdim, n, seed=dim + heads, rot=rot, norm=form != "plain", **FORMS[form])
    if form == "plain":
        gate = None
    want = ranged_oracle(q, k, v, gate, p, kv_heads, dim, vdim)
    kv = runtime.RangedKVCache(hip, 1, kv_heads, dim, vdim, 16, 192, elem)
    for cuts in ([n], [2, 3, 16, 31, 33, 2, 64], [1] * n):
        kv.reset()
        got = in_portions(n, cuts, lambda a, b: kv.attend(0, p, q[a:b], k[a:b], v[a:b], None if gate is None else gate[a:b]))
        assert kv.length(0) == n and rel(got, want) < TOL[elem], cuts[:3]
    kv.free()


@pytest.mark.parametrize("elem", [F16, F32])
@pytest.mark.parametrize("kind,size", [("window", 64), ("window", 65), ("window", 96), ("chunk", 64), ("chunk", 100), ("chunk", 33)])
def test_a_key_at_the_edge_of_a_range_stands_out(hip, kind, size, elem):
    """Query 199 and query 200 match one key so well that it takes nearly all the weight -- if it is in their range: at both sides of the edge, at
    page and tile borders, the first tokens of the range and of the sequence, in prompts and as single tokens."""
    heads, kv_heads, dim, vdim, n = 4, 2, 24, 40, 201
    q, k, v, gate, p = ranged_case(heads, kv_heads, dim, vdim, n, seed=5, mask=(kind, size), norm=False, scale=0.6, softcap=20.0, sink=1)
    edge = [max(0, i - size + 1) if kind == "window" else i // size * size for i in (199, 200)]
    q[199:] = 0
    kv = runtime.RangedKVCache(hip, 1, kv_heads, dim, vdim, 16, 224, elem)
    for far in sorted({0, 1, *(e + d for e in edge for d in (-2, -1, 0, 1)), 127, 128, 143, 144, 159, 160, 191, 192, 198}):
        if not 0 <= far < 199:
            continue
        qq, kk = q.copy(), k.copy()
        qq[199:] = np.tile(k[far].reshape(kv_heads, dim).repeat(heads // kv_heads, 0).reshape(-1), (2, 1)) * 2
        want = ranged_oracle(qq, kk, v, gate, p, kv_heads, dim, vdim)
        gone = kk.copy()
        gone[far] *= -1
        without = ranged_oracle(qq, gone, v, gate, p, kv_heads, dim, vdim)
        for i in (199, 200):
            shows = np.abs(want[i] - without[i]).max() > 0.2 * np.abs(want[i]).max()
            assert shows == (far >= edge[i - 199])
        for cuts in ([n], [199, 1, 1], [far + 1, n - far - 1], [150, 51]):
            kv.reset()
            got = in_portions(n, cuts, lambda a, b: kv.attend(0, p, qq[a:b], kk[a:b], v[a:b], gate[a:b]))
            assert rel(got[199:], want[199:]) < TOL[elem], (far, cuts)
    kv.free()


def test_pages_that_are_freed_and_used_again_by_other_sequences(hip):
    heads, kv_heads, dim, vdim = 4, 2, 48, 32
    kv = runtime.RangedKVCache(hip, 3, kv_heads, dim, vdim, 8, 64)
    cases = {s: ranged_case(heads, kv_heads, dim, vdim, n, seed=40 + s, mask=("window", 13), rot=16) for s, n in ((0, 50), (1, 17), (2, 33))}
    for turn in range(3):
        order = [0, 1, 2] if turn % 2 == 0 else [2, 0, 1]
        for s in order:  # (three sequences grow in turns, then one is dropped and starts again)
            q, k, v, gate, p = cases[s]
            kv.reset(s)
            half = len(q) // 2
            a = kv.attend(s, p, q[:half], k[:half], v[:half], gate[:half])
            other = order[(order.index(s) + 1) % 3]
            if kv.length(other):
                kv.reset(other)
            b = kv.attend(s, p, q[half:], k[half:], v[half:], gate[half:])
            assert rel(np.concatenate([a, b]), ranged_oracle(q, k, v, gate, p, kv_heads, dim, vdim)) < TOL[F16], (turn, s)
    kv.free()


# ---- attention over latents --------------------------------------------------------------------------------------------------

def latent_case(heads, dim, rot, vdim, rank, n, seed, mask=None, bf16=True, scale=None):
    rng = np.random.default_rng(seed)
    w = {"uk": rng.standard_normal((heads * dim, rank)).astype(np.float32) * rank ** -0.5, "uv": rng.standard_normal((heads * vdim, rank)).astype(np.float32) * rank ** -0.5}
    w = {name: bf16_to_f32(f32_to_bf16(a)) for name, a in w.items()}
    pk = Packer(lambda name: w[name], runtime.BF16 if bf16 else F32)
    p = {"n_head": heads, "dim": dim, "vdim": vdim, "scale": 2 * (dim + rot) ** -0.5 if scale is None else scale, "eps": 1e-5, "mask": mask, "rot_base": 700.0,
         "norm": (1 + 0.3 * rng.standard_normal(rank)).astype(np.float32), "w_up": pk.stack([("uk", heads * dim), ("uv", heads * vdim)], rank)}
    q = rng.standard_normal((n, heads * (dim + rot))).astype(np.float32)
    d = (2 * rng.standard_normal((n, rank + rot))).astype(np.float32)
    return q, d, p, w


def latent_oracle(q, d, p, w, rot, rank):
    n, H, D = len(q), p["n_head"], p["dim"]
    q, d = q.astype(np.float64).reshape(n, H, D + rot), d.astype(np.float64)
    c = orc.plain_norm(d[:, :rank], p["norm"].astype(np.float64), p["eps"])
    k_rot, q_rot = (orc.rotate_half(a, np.arange(n), p["rot_base"], rot) for a in (d[:, rank:], q[..., D:]))
    k, v = (c @ w["uk"].T).reshape(n, H, D), (c @ w["uv"].T).reshape(n, H, -1)
    s = (np.einsum("thd,shd->hts", q[..., :D], k) + np.einsum("thd,sd->hts", q_rot, k_rot)) * p["scale"]
    return np.einsum("hts,shv->thv", orc.softmax(s, mask_of(p, n)), v).reshape(n, -1)


LATENTS = [(4, 32, 32, 64, 64), (3, 24, 8, 20, 40), (2, 64, 64, 128, 200), (2, 128, 64, 128, 512), (2, 100, 20, 250, 70), (1, 200, 100, 33, 900), (1, 1, 2, 1, 1)]
LATENT_TOL = {F16: 1.5e-2, F32: 5e-6}  # (16-bit prompts round latents, keys and values once each)


@pytest.mark.parametrize("elem", [F16, F32])
@pytest.mark.parametrize("mask", [None, ("window", 33), ("chunk", 50)])
@pytest.mark.parametrize("heads,dim,rot,vdim,rank", LATENTS)
def test_latent_attention_in_one_go_in_portions_and_token_by_token(hip, heads, dim, rot, vdim, rank, mask, elem):
    n = 110
    q, d, p, w = latent_case(heads, dim, rot, vdim, rank, n, seed=rank + heads, mask=mask, bf16=elem == F16)
    want = latent_oracle(q, d, p, w, rot, rank)
    kv = runtime.LatentKVCache(hip, 1, rank, rot, 16, 128, elem)
    for cuts in ([n], [2, 3, 16, 31, 33, 2, 64], [1] * n):
        kv.reset()
        got = in_portions(n, cuts, lambda a, b: kv.attend(0, p, q[a:b], d[a:b]))
        assert kv.length(0) == n and rel(got, want) < LATENT_TOL[elem], cuts[:3]
    kv.free()


@pytest.mark.parametrize("elem", [F16, F32])
def test_latents_read_again_by_other_heads(hip, elem):
    rot, rank, n = 16, 56, 90
    q, d, p, w = latent_case(3, 24, rot, 40, rank, n, seed=1, mask=("window", 20), bf16=elem == F16)
    q2, _, p2, w2 = latent_case(5, 40, rot, 16, rank, n, seed=2, mask=("window", 31), bf16=elem == F16)
    p2["norm"] = p["norm"]
    want, want2 = latent_oracle(q, d, p, w, rot, rank), latent_oracle(q2, d, p2, w2, rot, rank)
    kv = runtime.LatentKVCache(hip, 1, rank, rot, 8, 96, elem)
    for cuts in ([n], [40, 2, 48], [60] + [1] * 30):
        kv.reset()

        def both(a, b):
            x = kv.attend(0, p, q[a:b], d[a:b])
            return np.concatenate([x, kv.attend(0, {**p2, "norm": None}, q2[a:b])], axis=1)

        got = in_portions(n, cuts, both)
        assert rel(got[:, :120], want) < LATENT_TOL[elem] and rel(got[:, 120:], want2) < LATENT_TOL[elem] and kv.length(0) == n
    kv.free()


@pytest.mark.parametrize("elem", [F16, F32])
@pytest.mark.parametrize("size", [64, 65, 96])
def test_a_latent_at_the_edge_of_a_window_stands_out(hip, size, elem):
    heads, dim, rot, vdim, rank, n = 2, 32, 8, 24, 40, 201
    q, d, p, w = latent_case(heads, dim, rot, vdim, rank, n, seed=9, mask=("window", size), bf16=elem == F16, scale=0.4)
    kv = runtime.LatentKVCache(hip, 1, rank, rot, 16, 224, elem)
    q[199:] = 0
    for far in sorted({0, 1, *(i - size + 1 + e for i in (199, 200) for e in (-2, -1, 0, 1)), 143, 144, 159, 160, 198}):
        qq = q.copy()
        c = orc.plain_norm(d[far, :rank].astype(np.float64), p["norm"].astype(np.float64), p["eps"])
        qq[199:].reshape(2, heads, dim + rot)[..., :dim] = 2 * (c @ w["uk"].T).reshape(heads, dim)
        want = latent_oracle(qq, d, p, w, rot, rank)
        gone = d.copy()
        gone[far] *= -1
        without = latent_oracle(qq, gone, p, w, rot, rank)
        for i in (199, 200):
            assert (np.abs(want[i] - without[i]).max() > 0.2 * np.abs(want[i]).max()) == (far > i - size)
        for cuts in ([n], [199, 1, 1], [far + 1, n - far - 1], [150, 51]):
            kv.reset()
            got = in_portions(n, cuts, lambda a, b: kv.attend(0, p, qq[a:b], d[a:b]))
            assert rel(got[199:], want[199:]) < LATENT_TOL[elem], (far, cuts)
    kv.free()


def test_cache_errors(hip):
    kv = runtime.RangedKVCache(hip, 1, 2, 32, 16, 8, 16)
    q, k, v, gate, p = ranged_case(4, 2, 32, 16, 17, seed=1)
    with pytest.raises(runtime.SknError) as e:
        kv.attend(0, p, q, k, v)
    assert e.value.code == runtime.ERR_POOL
    for bad in ({"n_head": 3}, {"rot_dims": 34}, {"rot_dims": 3}, {"mask": ("window", 0)}):
        with pytest.raises(runtime.SknError):
            kv.attend(0, {**p, **bad}, q[:2], k[:2], v[:2])
    buf = hip.alloc(1 << 16)
    assert hip.lib.skn_attn_decode(hip.handle, kv.handle, buf.ptr, None, 1.0, buf.ptr) == runtime.ERR_STATE
    assert hip.lib.skn_kv_append_run(hip.handle, kv.handle, 0, buf.ptr, buf.ptr, 1) == runtime.ERR_STATE
    kv.free()
    kv = runtime.LatentKVCache(hip, 1, 40, 8, 8, 16)
    q, d, p, _ = latent_case(2, 16, 8, 16, 40, 3, seed=1)
    with pytest.raises(runtime.SknError) as e:
        kv.attend(0, p, q)  # nothing is there to be read again
    assert e.value.code == runtime.ERR_RANGE
    with pytest.raises(runtime.SknError):
        kv.attend(0, {**p, "norm": None}, q, d)
    kv.free()
    for make in (lambda: runtime.RangedKVCache(hip, 1, 2, 257, 8, 8, 16), lambda: runtime.LatentKVCache(hip, 1, 1000, 32, 8, 16),
                 lambda: runtime.LatentKVCache(hip, 1, 64, 7, 8, 16), lambda: runtime.ConvRecurrentState(hip, 1, 4, 3, 8, 8, 4),
                 lambda: runtime.ConvRecurrentState(hip, 1, 4, 2, 8, 8, 9), lambda: runtime.ConvRecurrentState(hip, 1, 1, 1, 8, 257, 4)):
        with pytest.raises(runtime.SknError):
            make()


# ---- gated delta rule ----------------------------------------------------------------------------------------------------------

def delta_case(heads, kv_heads, dim, vdim, taps, n, seed, spread=3.0, shift=-1.0):
    rng = np.random.default_rng(seed)
    f = lambda *s: rng.standard_normal(s).astype(np.float32)  # noqa: E731
    return {"conv": f(2 * kv_heads * dim + heads * vdim, taps), "rate": np.exp(rng.uniform(-3, 2.5, heads)).astype(np.float32), "q": f(n, kv_heads * dim),
            "k": f(n, kv_heads * dim), "v": f(n, heads * vdim), "beta": orc.sigmoid(2 * f(n, heads)).astype(np.float32), "z": spread * f(n, heads * dim) + np.float32(shift)}


def delta_oracle(c, heads, kv_heads, dim, vdim):
    n, qk = len(c["q"]), kv_heads * dim
    d = {k: v.astype(np.float64) for k, v in c.items()}
    q, k, v = (orc.silu(orc.causal_conv(d[x], d["conv"][a:b])) for x, a, b in (("q", 0, qk), ("k", qk, 2 * qk), ("v", 2 * qk, None)))
    of = np.arange(heads) // (heads // kv_heads)
    q, k = (orc.unit(x.reshape(n, kv_heads, dim))[:, of] for x in (q, k))
    decay = np.exp(-d["rate"][:, None] * orc.softplus(d["z"].reshape(n, heads, dim)))
    return orc.gated_delta_rule(q * dim ** -0.5, k, v.reshape(n, heads, vdim), decay, d["beta"])[0].reshape(n, -1)


def advance(st, c, a, b, seq=0):
    return st.advance(seq, c["conv"], c["rate"], *(c[x][a:b] for x in ("q", "k", "v", "beta", "z")))


DELTAS = [(1, 1, 1, 1, 1), (2, 1, 5, 9, 2), (3, 3, 16, 16, 4), (4, 2, 32, 64, 3), (3, 1, 33, 20, 4), (2, 2, 64, 64, 8), (2, 1, 100, 256, 4), (1, 1, 128, 128, 5),
          (1, 1, 200, 48, 2), (1, 1, 256, 256, 4)]


@pytest.mark.parametrize("heads,kv_heads,dim,vdim,taps", DELTAS)
def test_gated_delta_in_one_go_in_portions_and_token_by_token(hip, heads, kv_heads, dim, vdim, taps):
    n = 70
    c = delta_case(heads, kv_heads, dim, vdim, taps, n, seed=dim)
    want = delta_oracle(c, heads, kv_heads, dim, vdim)
    st = runtime.ConvRecurrentState(hip, 1, heads, kv_heads, dim, vdim, taps)
    for cuts in ([n], [2, 3, 16, 15, 17, 1, 16], [1] * 20 + [50]):
        st.reset()
        assert rel(in_portions(n, cuts, lambda a, b: advance(st, c, a, b)), want) < 1e-5, cuts
    st.free()


def test_decays_from_nothing_to_everything(hip):
    """Some channels forget everything in one token, others nothing over hundreds; both change from token to token."""
    heads, kv_heads, dim, vdim, taps, n = 2, 1, 48, 32, 4, 400
    c = delta_case(heads, kv_heads, dim, vdim, taps, n, seed=7, spread=0.0, shift=0.0)
    rng = np.random.default_rng(8)
    c["z"] = rng.choice(np.float32([-40, -12, -3, 0, 4, 60, 300]), size=c["z"].shape, p=[0.3, 0.4, 0.2, 0.06, 0.02, 0.01, 0.01])
    want = delta_oracle(c, heads, kv_heads, dim, vdim)
    st = runtime.ConvRecurrentState(hip, 1, heads, kv_heads, dim, vdim, taps)
    got = advance(st, c, 0, n)
    assert np.all(np.isfinite(got)) and rel(got, want) < 2e-5
    st.reset()
    assert rel(in_portions(n, [100, 7, 290, 3], lambda a, b: advance(st, c, a, b)), want) < 2e-5
    st.free()


def test_it_remembers_over_a_long_sequence(hip):
    """Factors near one and small rates: the first token's value is still there a thousand tokens later."""
    heads, kv_heads, dim, vdim, taps, n = 2, 2, 24, 24, 4, 1000
    c = delta_case(heads, kv_heads, dim, vdim, taps, n, seed=3, spread=0.5, shift=-14.0)
    c["beta"] *= 0.02
    want = delta_oracle(c, heads, kv_heads, dim, vdim)
    other = {**c, "v": c["v"].copy()}
    other["v"][0] += 200
    assert rel(delta_oracle(other, heads, kv_heads, dim, vdim)[-1], want[-1]) > 1e-2
    st = runtime.ConvRecurrentState(hip, 1, heads, kv_heads, dim, vdim, taps)
    assert rel(advance(st, c, 0, n), want) < 2e-5
    st.free()


def test_states_of_several_sequences_stay_apart_and_reset(hip):
    shape = (2, 1, 40, 24)
    a, b = delta_case(*shape, 4, 20, seed=1), delta_case(*shape, 4, 31, seed=2)
    b = {**b, "conv": a["conv"], "rate": a["rate"]}
    wa, wb = delta_oracle(a, *shape), delta_oracle(b, *shape)
    st = runtime.ConvRecurrentState(hip, 3, *shape, 4)
    for _ in range(2):
        x0, y0 = advance(st, a, 0, 9), advance(st, b, 0, 11, 2)
        x1, y1 = advance(st, a, 9, 20), advance(st, b, 11, 31, 2)
        assert rel(np.concatenate([x0, x1]), wa) < 1e-5 and rel(np.concatenate([y0, y1]), wb) < 1e-5
        st.reset(0)
        assert rel(advance(st, a, 0, 20), wa) < 1e-5
        st.reset()
    st.free()


def test_many_heads(hip):
    shape = (80, 16, 64, 64)
    c = delta_case(*shape, 4, 33, seed=9)
    st = runtime.ConvRecurrentState(hip, 1, *shape, 4)
    assert rel(advance(st, c, 0, 33), delta_oracle(c, *shape)) < 1e-5
    st.free()
