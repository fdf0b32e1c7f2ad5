"""Cases of the decoder blocks (the last section of include/catgrad_hip.h), run on the CPU oracle and on the HIP library
against the plain statements of loretar_reference.py."""
import numpy as np

import loretar_reference as R
from catgrad_amd import BF16


def bf16(x):
    """float32 values rounded to bfloat16 (nearest, ties to even)."""
    u = np.ascontiguousarray(x, dtype=np.float32).view(np.uint32)
    u = (u + 0x7FFF + ((u >> 16) & 1)) & np.uint32(0xFFFF0000)
    return u.view(np.float32)


def weight(be, w, dtype):
    t = be.from_numpy(np.ascontiguousarray(w, dtype=np.float32))
    return t if dtype == "f32" else be.cast(t, BF16)


def close(got, want, tol, what=""):
    scale = np.sqrt((np.asarray(want) ** 2).mean()) + 1e-30
    err = np.abs(got - want).max() / scale
    assert err <= tol, f"{what}: largest error {err:.3g} of the result's scale, allowed {tol:.3g}"


def part_of_rows(be, x, before=8, behind=5):
    """x [.., n] as a view of the columns before .. before + n of wider rows."""
    wide = np.concatenate([np.full(x.shape[:-1] + (before,), 7.0), x, np.full(x.shape[:-1] + (behind,), -9.0)], -1).astype(np.float32)
    return be.slice(be.from_numpy(wide), x.ndim - 1, before, x.shape[-1])


# ---- products --------------------------------------------------------------------------------------------------------
LINEAR = [  # rows, K of x, K of x2, N, weight dtype, RMS norm, bias, view
    (1, 24, 0, 7, "f32", False, False, False), (1, 257, 0, 96, "f32", True, False, False), (3, 40, 0, 300, "f32", True, True, True),
    (5, 512, 0, 1030, "f32", True, False, False), (8, 2048, 0, 96, "f32", True, False, False), (1, 1024, 0, 8200, "f32", True, False, False),
    (2, 520, 0, 4100, "bf16", True, True, True), (1, 1024, 0, 8200, "bf16", True, False, False), (4, 2048, 0, 4100, "bf16", True, False, True),
    (8, 4096, 0, 300, "bf16", True, False, False), (7, 1536, 1536, 130, "bf16", False, True, False), (1, 48, 48, 48, "f32", False, True, False),
    (2, 33, 65, 50, "bf16", True, True, True), (1, 96, 0, 700, "bf16", False, False, False), (9, 257, 0, 96, "f32", True, True, True),
    (70, 96, 96, 130, "f32", False, True, False), (70, 512, 0, 520, "bf16", True, False, True), (300, 256, 0, 264, "bf16", True, True, False),
    (520, 1024, 0, 1040, "bf16", True, False, False), (1, 30000, 0, 20, "f32", True, False, False),
    (9, 1032, 0, 260, "bf16", False, False, False), (64, 520, 0, 388, "bf16", False, True, False), (65, 776, 0, 257, "bf16", False, False, True),
    (129, 2088, 0, 132, "bf16", False, False, False), (200, 264, 256, 640, "bf16", True, False, False), (33, 8, 0, 9000, "bf16", False, False, False),
    (1000, 1024, 0, 5000, "bf16", False, False, False), (300, 4096, 0, 516, "bf16", False, True, False)]


def run_linear(be, case, seed=0):
    rows, k1, k2, n, dt, norm, bias, view = case
    rng = np.random.default_rng(seed)
    x, x2 = rng.standard_normal((1, rows, k1)).astype(np.float32), rng.standard_normal((1, rows, k2)).astype(np.float32)
    K = k1 + k2
    w = bf16(rng.standard_normal((n, K)) * K ** -0.5)
    exact = dt == "f32" or not norm  # (the operand has its values before the product rounds them)
    if dt == "bf16" and exact:
        x, x2 = bf16(x), bf16(x2)
    gamma, b = (1 + 0.3 * rng.standard_normal(K)).astype(np.float32), rng.standard_normal(n).astype(np.float32)
    eps, scale = 3e-3, 0.7
    xt = part_of_rows(be, x) if view else be.from_numpy(x)
    out = be.block_linear(xt, weight(be, w, dt), x2=be.from_numpy(x2) if k2 else None, gamma=be.from_numpy(gamma) if norm else None,
                          bias=be.from_numpy(b) if bias else None, eps=eps, scale=scale)
    ref = np.concatenate([x, x2], -1)[0].astype(np.float64)
    if norm:
        ref = R.rms_norm(ref, gamma.astype(np.float64), eps)
    ref = ref @ w.T.astype(np.float64) * scale + (b if bias else 0.0)
    assert out.shape == (1, rows, n)
    close(be.to_numpy(out)[0], ref, 2e-5 if exact else 2e-2, f"linear {case}")


RESIDUAL = [  # rows, width, [(K, poly, gate)], weight dtype
    (1, 64, [(40, False, True), (96, True, True)], "f32"), (1, 520, [(257, True, False)], "f32"), (2, 256, [(512, False, True), (768, True, True)], "bf16"),
    (4, 2048, [(2048, False, True), (8192, True, True)], "f32"), (4, 1024, [(1024, False, True), (6144, True, True)], "bf16"),
    (8, 96, [(48, False, True), (130, True, True)], "bf16"), (3, 130, [(48, False, True), (52, True, False)], "bf16"),
    (1, 4096, [(48, False, True), (512, True, True)], "bf16"), (9, 64, [(40, False, True), (96, True, True)], "f32"),
    (70, 256, [(512, False, True), (768, True, True)], "bf16"), (33, 130, [(52, False, False), (48, True, True)], "f32"), (65, 96, [(64, False, True)], "f32")]


def run_residual(be, case, seed=0):
    rows, width, parts, dt = case
    rng = np.random.default_rng(seed)
    eps = 2e-3
    x = rng.standard_normal((1, rows, width)).astype(np.float32)
    ref, br = x[0].astype(np.float64), []
    for i, (K, poly, gate) in enumerate(parts):
        y, w = rng.standard_normal((1, rows, K)).astype(np.float32), bf16(rng.standard_normal((width, K)) * K ** -0.5)
        g, gb = rng.standard_normal((1, rows, width)).astype(np.float32), rng.standard_normal(width).astype(np.float32)
        c = rng.standard_normal(4).astype(np.float32)
        d = {"y": part_of_rows(be, y) if i else be.from_numpy(y), "w": weight(be, w, dt)}
        z = y[0].astype(np.float64)
        if poly:
            d["poly"] = be.from_numpy(c)
            z = R.poly_norm(z, c.astype(np.float64), eps)
        z = z @ w.T.astype(np.float64)
        if gate:
            d["gate"], d["gate_bias"] = part_of_rows(be, g), be.from_numpy(gb)
            z = z * R.sigmoid((g[0] + gb).astype(np.float64))
        br.append(d)
        ref = ref + z
    out = be.block_residual(be.from_numpy(x), br, eps)
    close(be.to_numpy(out)[0], ref, 2e-5 if dt == "f32" else 2e-2, f"residual {case}")


# ---- attention -------------------------------------------------------------------------------------------------------
def attention_reference(q, k, v, o, qn=None, kn=None, talk=None):
    """One sequence: raw projections [S, ..] -> [S, heads * vdim]."""
    S, H, G = q.shape[0], o["heads"], o["kv_heads"]
    q, k, v = q.astype(np.float64), k.astype(np.float64), v.astype(np.float64)
    if qn is not None:
        q = R.rms_norm(q, qn.astype(np.float64), o["norm_eps"])
    if kn is not None:
        k = R.rms_norm(k, kn.astype(np.float64), o["norm_eps"])
    if o.get("temp_every"):
        q = q * R.query_temperature(np.arange(S), o["temp_coef"], o["temp_every"])[:, None]
    q = q.reshape(S, H, -1).transpose(1, 0, 2)
    k, v = k.reshape(S, G, -1).transpose(1, 0, 2), v.reshape(S, G, -1).transpose(1, 0, 2)
    w = R.attention_weights(q, k, o["scale"], R.alibi_slopes(H) if o.get("distance_bias") else None, o.get("window") or None)
    if talk is not None:
        w = np.tensordot(talk.astype(np.float64), w, axes=(1, 0))
    return np.stack([w[h] @ v[h // (H // G)] for h in range(H)], 1).reshape(S, -1)


def attention_case(rng, B, S, o, norms=True, talk=True):
    H, G, D, V = o["heads"], o["kv_heads"], o["dim"], o["vdim"]
    t = {"q": rng.standard_normal((B, S, H * D)), "k": rng.standard_normal((B, S, G * D)), "v": rng.standard_normal((B, S, G * V))}
    if norms:
        t["q_norm"], t["k_norm"] = 1 + 0.3 * rng.standard_normal(H * D), 1 + 0.3 * rng.standard_normal(G * D)
    if talk:
        t["talk"] = np.eye(H) + 0.5 * rng.standard_normal((H, H))
    return {n: a.astype(np.float32) for n, a in t.items()}


def run_attention(be, t, o, portions):
    """The sequence in portions of these lengths, through the cache: [B, S, heads * vdim]."""
    B = t["q"].shape[0]
    kc, vc = be.zeros((B, o["kv_heads"], 0, o["dim"]), 0), be.zeros((B, o["kv_heads"], 0, o["vdim"]), 0)
    small = {n: be.from_numpy(t[n]) for n in ("q_norm", "k_norm", "talk") if n in t}
    at, outs = 0, []
    for n in portions:
        part = {c: part_of_rows(be, t[c][:, at:at + n]) for c in ("q", "k", "v")}
        out, kc, vc = be.block_attention({**part, **small, "k_cache": kc.move(), "v_cache": vc.move()}, position=at, **o)
        at += n
        w = o.get("window")
        assert kc.shape[2] == vc.shape[2] == (min(at, w - 1) if w else at)
        outs.append(be.to_numpy(out))
    assert at == t["q"].shape[1]
    return np.concatenate(outs, 1)


def check_attention(be, t, o, portions, tol=3e-5):
    got = run_attention(be, t, o, portions)
    for b in range(t["q"].shape[0]):
        want = attention_reference(t["q"][b], t["k"][b], t["v"][b], o, t.get("q_norm"), t.get("k_norm"), t.get("talk"))
        close(got[b], want, tol, f"attention {o}, portions {portions[:6]}, sequence {b}")


def options(heads, kv_heads, dim, vdim, window, **kw):
    o = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, window=window, scale=dim ** -0.5, norm_eps=1e-3, temp_coef=0.3, temp_every=7,
             distance_bias=1)
    o.update(kw)
    return o


ATTENTION = {  # name: (options, batch, portions, norms, talk)
    "whole": (options(4, 2, 16, 16, 9), 1, [40], True, True),
    "one_head": (options(1, 1, 8, 12, 5), 1, [20, 3, 1, 1], True, True),
    "token_by_token": (options(4, 4, 16, 20, 6), 2, [1] * 20, True, True),
    "odd_sizes": (options(6, 2, 10, 7, 11), 1, [13, 2, 30, 1, 1, 9], True, True),
    "three_heads": (options(3, 1, 12, 20, 17), 2, [50, 2, 5, 1], True, True),
    "many_heads": (options(24, 4, 32, 16, 33), 1, [70, 1, 1, 20], True, True),
    "more_heads_than_tiles_take": (options(40, 8, 8, 8, 20), 1, [30, 1, 10], True, True),
    "ten_per_kv_head": (options(10, 1, 8, 8, 20), 1, [30, 1, 2], True, True),
    "wide": (options(4, 2, 128, 96, 40), 1, [64, 1, 33], True, True),
    "wider_than_tiles_take": (options(2, 1, 160, 144, 40), 1, [30, 1, 12], True, True),
    "window_1": (options(4, 2, 16, 16, 1), 1, [12, 1, 1, 4], True, True),
    "window_2": (options(4, 2, 16, 16, 2), 1, [12, 1, 1, 4], True, True),
    "no_window": (options(4, 2, 16, 16, 0), 1, [40, 1, 1, 10, 30], True, True),
    "window_of_the_prompt": (options(4, 2, 32, 32, 64), 1, [64, 1, 1, 1], True, True),
    "window_longer_than_all": (options(4, 2, 32, 32, 500), 1, [64, 1, 40], True, True),
    "no_talk": (options(8, 2, 32, 32, 21), 2, [45, 1, 9, 12], True, False),
    "no_norms": (options(8, 4, 32, 48, 21), 1, [45, 1, 9, 12], False, True),
    "nothing": (options(8, 4, 64, 64, 0, distance_bias=0, temp_every=0), 1, [45, 1, 12], False, False),
    "no_bias": (options(4, 2, 16, 16, 30, distance_bias=0), 1, [50, 1], True, True),
    "no_temperature": (options(4, 2, 16, 16, 30, temp_every=0), 1, [50, 1], True, True),
    "segments_of_keys": (options(4, 1, 16, 16, 300), 1, [400, 1, 1, 5], True, True),
    "long_prompt_then_decode": (options(2, 1, 16, 16, 40), 1, [700] + [1] * 12, True, True),
    "keys_cut_over_workgroups": (options(16, 4, 64, 64, 600), 1, [640, 100], True, True),
}


def run_attention_case(be, name):
    o, B, portions, norms, talk = ATTENTION[name]
    rng = np.random.default_rng(sum(map(ord, name)))
    check_attention(be, attention_case(rng, B, sum(portions), o, norms, talk), o, portions)


def run_attention_edges(be, window, portions, dim=16):
    """One key stands out for one query, just inside or just outside the window, or far behind: the weights of that row then
    show whether it was seen."""
    S = sum(portions)
    o = options(4, 2, dim, 16, window, distance_bias=0, temp_every=0)
    rng = np.random.default_rng(window)
    starts = np.cumsum([0] + portions)[:-1]
    rows = sorted({int(i) for s in starts for i in (s, s + 1, s - 1) if 0 <= i < S} | {S - 1, window - 1, window, window + 1} & set(range(S)))
    for i in rows:
        for back in (window - 1, window, window + 1, 1, 0):
            j = i - back
            if j < 0:
                continue
            t = attention_case(rng, 1, S, o, norms=False)
            for g in range(2):  # both kv heads' key j points along the queries of row i
                t["k"][0, j, g * dim:(g + 1) * dim] = 6.0
            t["q"][0, i] = 2.0
            got = run_attention(be, t, o, portions)[0, i]
            want = attention_reference(t["q"][0], t["k"][0], t["v"][0], o, None, None, t["talk"])[i]
            close(got, want, 1e-4, f"window {window}, row {i} looking {back} back, portions {portions}")


# ---- gated delta rule ------------------------------------------------------------------------------------------------
def delta_case(rng, B, S, o, taps, r1, r2, decay_at=-3.0):
    H, G, D, V = o["heads"], o["kv_heads"], o["dim"], o["vdim"]
    n = rng.standard_normal
    t = {"q": n((B, S, G * D)), "k": n((B, S, G * D)), "v": n((B, S, H * V)), "conv_q": n((G * D, taps)) * taps ** -0.5,
         "conv_k": n((G * D, taps)) * taps ** -0.5, "conv_v": n((H * V, taps)) * taps ** -0.5, "beta": n((B, S, H)), "decay": n((B, S, r1)),
         "decay_w": n((H * D, r1)) * r1 ** -0.5, "a_log": 0.5 * n(H), "dt_bias": n(H * D) + decay_at, "gate": n((B, S, r2)),
         "gate_w": n((H * V, r2)) * r2 ** -0.5, "norm": 1 + 0.3 * n(V)}
    return {k: v.astype(np.float32) for k, v in t.items()}


def delta_reference(t, b, o):
    """Sequence b: (output [S, heads * vdim], final state [heads, dim, vdim], last inputs of the convolutions)."""
    H, G, D, V = o["heads"], o["kv_heads"], o["dim"], o["vdim"]
    t = {k: v.astype(np.float64) for k, v in t.items()}
    S = t["q"].shape[1]

    def conv(x, c, heads):
        return R.silu(R.short_conv(x[b], c)).reshape(S, heads, -1)

    q, k, v = conv(t["q"], t["conv_q"], G), conv(t["k"], t["conv_k"], G), conv(t["v"], t["conv_v"], H)
    q, k = np.repeat(R.unit(q) * D ** -0.5, H // G, 1), np.repeat(R.unit(k), H // G, 1)
    g = R.channel_decay(t["decay"][b] @ t["decay_w"].T, t["a_log"], t["dt_bias"], H, D)
    y, state = R.delta_rule(q, k, v, R.sigmoid(t["beta"][b]), g)
    y = R.rms_norm(y, t["norm"], o["eps"]) * R.sigmoid(t["gate"][b] @ t["gate_w"].T).reshape(S, H, V)
    taps = t["conv_q"].shape[1]
    raw = np.concatenate([t["q"][b], t["k"][b], t["v"][b]], -1)
    raw = np.concatenate([np.zeros((taps - 1, raw.shape[1])), raw])
    return y.reshape(S, -1), state, raw[S:]


def run_delta(be, t, o, portions):
    B, taps = t["q"].shape[0], t["conv_q"].shape[1]
    H, G, D, V = o["heads"], o["kv_heads"], o["dim"], o["vdim"]
    state, conv = be.zeros((B, H, D, V), 0), be.zeros((B, taps - 1, 2 * G * D + H * V), 0)
    seq = ("q", "k", "v", "beta", "decay", "gate")
    small = {n: be.from_numpy(a) for n, a in t.items() if n not in seq}
    at, outs = 0, []
    for n in portions:
        part = {c: part_of_rows(be, t[c][:, at:at + n]) for c in seq}
        out, state, conv = be.block_channel_delta({**part, **small, "state": state.move(), "conv_state": conv.move()}, **o)
        at += n
        outs.append(be.to_numpy(out))
    return np.concatenate(outs, 1), be.to_numpy(state), be.to_numpy(conv)


def check_delta(be, t, o, portions, tol=1e-4):
    got, state, conv = run_delta(be, t, o, portions)
    for b in range(t["q"].shape[0]):
        want, s, c = delta_reference(t, b, o)
        close(got[b], want, tol, f"channel delta {o}, portions {portions[:6]}, sequence {b}")
        close(state[b], s, tol, f"state after {portions[:6]}")
        if c.size:
            np.testing.assert_allclose(conv[b], c, rtol=1e-6, atol=1e-6)


def delta_options(heads, kv_heads, dim, vdim):
    return dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, eps=1e-3)


DELTA = {  # name: (options, batch, taps, ranks, portions, dt_bias around)
    "whole": (delta_options(2, 2, 16, 16), 1, 4, (12, 9), [50], -3.0),
    "token_by_token": (delta_options(4, 2, 16, 24), 2, 4, (8, 8), [1] * 12, -3.0),
    "odd_sizes": (delta_options(3, 1, 10, 7), 1, 3, (5, 6), [17, 2, 1, 1, 20, 3], -3.0),
    "one_tap": (delta_options(2, 1, 16, 16), 1, 1, (8, 8), [20, 1, 2, 16], -3.0),
    "two_taps_short_portions": (delta_options(2, 2, 32, 32), 1, 2, (8, 8), [2, 2, 1, 3, 2, 16], -3.0),
    "long_taps": (delta_options(2, 2, 16, 16), 1, 6, (8, 8), [2, 1, 2, 3, 9, 1, 1, 40], -3.0),
    "one_head": (delta_options(1, 1, 40, 20), 2, 4, (16, 4), [33, 5], -3.0),
    "shared_keys": (delta_options(6, 2, 24, 48), 1, 4, (16, 16), [31, 1, 18], -3.0),
    "wide": (delta_options(2, 2, 128, 128), 1, 4, (64, 64), [70, 1, 16, 15, 1], -3.0),
    "widest": (delta_options(1, 1, 256, 64), 1, 4, (16, 16), [40, 1, 3], -3.0),
    "chunk_edges": (delta_options(2, 1, 64, 80), 2, 4, (8, 8), [16, 15, 17, 32, 1, 31, 9, 12], -3.0),
    "fast_decay": (delta_options(2, 2, 32, 32), 1, 4, (8, 8), [60, 1, 20], 6.0),
    "slow_decay": (delta_options(2, 2, 32, 32), 1, 4, (8, 8), [200, 1, 20], -12.0),
}


def run_delta_case(be, name):
    o, B, taps, ranks, portions, at = DELTA[name]
    rng = np.random.default_rng(sum(map(ord, name)))
    check_delta(be, delta_case(rng, B, sum(portions), o, taps, *ranks, decay_at=at), o, portions)
