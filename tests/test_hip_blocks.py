"""The decoder blocks on the GPU against the plain statements of loretar_reference.py and lufatar_reference.py."""
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


@pytest.mark.parametrize("name", list(C.MIXED))
def test_mixed_scores(hip, name):
    C.run_mixed_case(hip, name)


@pytest.mark.parametrize("portions", [[20, 1, 2, 17], [80, 1, 1, 2, 70], [140, 1, 3, 9, 1]], ids=str)
def test_mixed_scores_needles(hip, portions):
    C.run_mixed_needles(hip, C.turned(4, 2, 16, 16, 0), portions)


@pytest.mark.parametrize("dim,vdim", [(16, 16), (32, 20), (48, 96), (64, 64), (64, 80), (96, 48), (128, 128)])
@pytest.mark.parametrize("heads,kv_heads", [(4, 2), (8, 8), (12, 3), (16, 2), (20, 5), (32, 8), (32, 4)])
def test_mixed_scores_shapes(hip, heads, kv_heads, dim, vdim):
    """Every instantiation of the tiled and the step kernels: heads per wave, query heads per key head, widths."""
    rng = np.random.default_rng(heads * dim + vdim)
    o = C.turned(heads, kv_heads, dim, vdim, dim // 2 // 2 * 2)
    C.check_attention(hip, C.attention_case(rng, 1, 94, o, False, True), o, [41, 49, 1, 1, 2], tol=6e-5)


@pytest.mark.parametrize("dtype", ["f32", "bf16"])
def test_pair_embedding(hip, dtype):
    C.run_pair_embedding(hip, dtype)
    C.run_pair_embedding(hip, dtype, B=1, vocab=5000, buckets=4099, width=512, mul_prev=2 ** 40 + 9, mul_cur=2 ** 31 + 11)


@pytest.mark.parametrize("case", C.CONV, ids=str)
def test_conv_linear(hip, case):
    C.run_conv_linear(hip, case)


@pytest.mark.parametrize("case", [(3, 40, 5, 7, "f32"), (1, 2048, 4, 5000, "bf16"), (4, 1024, 8, 300, "f32"), (50, 96, 3, 130, "bf16"), (50, 30, 3, 13, "f32")], ids=str)
def test_grouped_linear(hip, case):
    C.run_grouped_linear(hip, *case)


@pytest.mark.parametrize("case", C.EXPERTS, ids=str)
def test_experts(hip, case):
    C.run_experts(hip, case)


@pytest.mark.parametrize("rows", [1, 5, 20, 300])
def test_expert_choices(hip, rows):
    C.run_expert_choices(hip, rows)


@pytest.mark.parametrize("case", C.SIDE, ids=str)
def test_token_side(hip, case):
    C.run_side(hip, case)


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
        C.run_mixed_case(hip, "twos_and_threes")
        for case in (C.CONV[2], C.CONV[9]):
            C.run_conv_linear(hip, case)
        for case in (C.EXPERTS[2], C.EXPERTS[10], C.EXPERTS[13]):
            C.run_experts(hip, case)
        for case in (C.SIDE[1], C.SIDE[5]):
            C.run_side(hip, case)

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
    ones = lambda *s: hip.from_numpy(np.ones(s, np.float32))
    ex = dict(h=x, logits=ones(1, 2, 4), gate_up=ones(4, 2, 6, 8), down=ones(4, 8, 6))
    for bad in (dict(top=5, groups=1, keep=1), dict(top=3, groups=2, keep=1), dict(top=2, groups=3, keep=1), dict(top=0, groups=1, keep=1), dict(top=2, groups=2, keep=3)):
        with pytest.raises(BackendPanic):
            hip.block_residual(x, [], experts=ex, **bad)
    with pytest.raises(BackendPanic):
        hip.block_residual(x, [], experts={**ex, "down": ones(4, 8, 5)}, top=2, groups=1, keep=1)
    with pytest.raises(BackendPanic):   # groups that do not divide the row
        hip.block_conv_linear(x, hip.zeros((1, 1, 8), 0), [{"gamma": ones(8), "conv": ones(8, 2), "w": ones(3, 8)}], groups=3)
    with pytest.raises(BackendPanic):
        hip.block_conv_linear(x, hip.zeros((1, 2, 8), 0), [{"gamma": ones(8), "conv": ones(8, 2), "w": ones(3, 8)}])
    with pytest.raises(BackendPanic):   # the table ends before the part
        hip.block_token_side(dict(x=x, ids=hip.from_numpy(np.zeros((1, 2), np.uint32)), table=ones(5, 8), gate=ones(4, 8), proj=ones(8, 4), norm=ones(8)), first=6)
