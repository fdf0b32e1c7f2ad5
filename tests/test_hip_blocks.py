"""The decoder blocks on the GPU against the plain statements of loretar_reference.py."""
import numpy as np
import pytest

import block_cases as C

pytestmark = pytest.mark.gpu


@pytest.mark.parametrize("case", C.LINEAR, ids=str)
def test_linear(hip, case):
    C.run_linear(hip, case)


@pytest.mark.parametrize("case", C.RESIDUAL, ids=str)
def test_residual(hip, case):
    C.run_residual(hip, case)


@pytest.mark.parametrize("name", list(C.ATTENTION))
def test_attention(hip, name):
    C.run_attention_case(hip, name)


@pytest.mark.parametrize("window,portions", [(5, [9, 1, 1, 6]), (16, [33, 1, 2, 12]), (33, [70, 1, 1, 20]), (130, [140, 1, 1, 9])])
def test_attention_edges(hip, window, portions):
    C.run_attention_edges(hip, window, portions)


@pytest.mark.parametrize("dim", [16, 32, 48, 64, 96, 128])
@pytest.mark.parametrize("heads,kv_heads", [(4, 2), (8, 8), (12, 3), (16, 2), (20, 5), (32, 8)])
def test_attention_tile_shapes(hip, heads, kv_heads, dim):
    """Every instantiation of the tiled kernels: heads per wave, widths of keys and values, with and without head mixing."""
    rng = np.random.default_rng(heads * dim)
    for vdim, talk in ((dim, True), (max(8, dim - 12), False)):
        o = C.options(heads, kv_heads, dim, vdim, 37)
        C.check_attention(hip, C.attention_case(rng, 1, 90, o, True, talk), o, [41, 49])


@pytest.mark.parametrize("name", list(C.DELTA))
def test_channel_delta(hip, name):
    C.run_delta_case(hip, name)


@pytest.mark.parametrize("dim", [8, 16, 24, 32, 64, 96, 128, 192, 256])
def test_channel_delta_key_widths(hip, dim):
    rng = np.random.default_rng(dim)
    o = C.delta_options(2, 1, dim, 40)
    C.check_delta(hip, C.delta_case(rng, 1, 60, o, 4, 8, 8), o, [37, 1, 2, 20])


def test_a_cache_that_two_continuations_share(hip):
    """Rows are appended behind the cache of a handle that somebody else still holds: both continuations see their own."""
    rng = np.random.default_rng(3)
    o = C.options(4, 2, 16, 16, 12)
    t = C.attention_case(rng, 1, 31, o)
    small = {n: hip.from_numpy(t[n]) for n in ("q_norm", "k_norm", "talk")}

    def step(src, lo, hi, kc, vc):
        part = {c: hip.from_numpy(src[c][:, lo:hi].copy()) for c in ("q", "k", "v")}
        return hip.block_attention({**part, **small, "k_cache": kc, "v_cache": vc}, position=lo, **o)

    other = {n: (a.copy() if n in small else np.concatenate([a[:, :30], -a[:, 30:]], 1)) for n, a in t.items()}
    _, kc, vc = step(t, 0, 30, hip.zeros((1, 2, 0, 16), 0), hip.zeros((1, 2, 0, 16), 0))
    a, ka, va = step(t, 30, 31, kc, vc)        # appended in place
    b, kb, vb = step(other, 30, 31, kc, vc)    # the same place is taken: a copy
    for got, src in ((a, t), (b, other)):
        want = C.attention_reference(src["q"][0], src["k"][0], src["v"][0], o, t["q_norm"], t["k_norm"], t["talk"])[30]
        C.close(hip.to_numpy(got)[0, 0], want, 3e-5)
    np.testing.assert_array_equal(hip.to_numpy(ka)[:, :, :-1], hip.to_numpy(kb)[:, :, :-1])


def test_blocks_give_their_memory_back(hip):
    rng = np.random.default_rng(4)
    o, d = C.options(4, 2, 16, 16, 9), C.delta_options(2, 2, 16, 16)
    t, u = C.attention_case(rng, 1, 60, o), C.delta_case(rng, 1, 60, d, 4, 8, 8)

    def once():
        C.run_attention(hip, t, o, [40, 1, 1, 18])
        C.run_delta(hip, u, d, [40, 1, 1, 18])
        C.run_linear(hip, C.LINEAR[2])
        C.run_residual(hip, C.RESIDUAL[2])

    once()
    hip.sync()
    before = hip.pool_stats()[0]
    for _ in range(3):
        once()
    hip.sync()
    assert hip.pool_stats()[0] == before


def test_misfits_are_errors(hip):
    from catgrad_amd import BackendPanic

    rng = np.random.default_rng(5)
    o = C.options(4, 2, 16, 16, 9)
    t = {n: hip.from_numpy(a) for n, a in C.attention_case(rng, 1, 4, o).items()}
    z = hip.zeros((1, 2, 0, 16), 0)
    with pytest.raises(BackendPanic):   # the cache does not reach back to the window
        hip.block_attention({**t, "k_cache": z, "v_cache": z}, position=6, **o)
    with pytest.raises(BackendPanic):
        hip.block_attention({**t, "k_cache": z, "v_cache": z}, position=0, **{**o, "kv_heads": 3})
    x = hip.from_numpy(rng.standard_normal((1, 2, 8)).astype(np.float32))
    with pytest.raises(BackendPanic):
        hip.block_linear(x, hip.from_numpy(np.ones((4, 9), np.float32)))
    with pytest.raises(BackendPanic):
        hip.block_residual(x, [{"y": x, "w": hip.from_numpy(np.ones((9, 8), np.float32))}])
