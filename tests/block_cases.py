"""Cases of the decoder blocks (the last section of include/catgrad_hip.h), run on the CPU oracle and on the HIP library
against the plain statements of loretar_reference.py and lufatar_reference.py."""
import numpy as np

import loretar_reference as R
import lufatar_reference as L
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
    q = q.reshape(S, H, -1).transpose(1, 0, 2)
    k, v = k.reshape(S, G, -1).transpose(1, 0, 2), v.reshape(S, G, -1).transpose(1, 0, 2)
    if o.get("rot_dims"):
        q, k = (L.rotate_pairs(x.transpose(1, 0, 2), np.arange(S), o["rot_base"], o["rot_dims"]).transpose(1, 0, 2) for x in (q, k))
    if o.get("unit_heads"):
        q, k = L.rms(q, o["norm_eps"]), L.rms(k, o["norm_eps"])
    if o.get("temp_every"):
        q = q * R.query_temperature(np.arange(S), o["temp_coef"], o["temp_every"])[:, None]
    if o.get("mix_scores") or o.get("zero_sink"):
        w = mixed_weights(q, k, o, talk if o.get("mix_scores") else None)
        talk = None if o.get("mix_scores") else talk
    else:
        w = R.attention_weights(q, k, o["scale"], R.alibi_slopes(H) if o.get("distance_bias") else None, o.get("window") or None)
    if talk is not None:
        w = np.tensordot(talk.astype(np.float64), w, axes=(1, 0))
    return np.stack([w[h] @ v[h // (H // G)] for h in range(H)], 1).reshape(S, -1)


def mixed_weights(q, k, o, talk):
    """Weights [H, S, S] of scores that talk mixes over the heads first, beside a score of 0 that goes nowhere, or neither."""
    H, S, _ = q.shape
    i, j = np.arange(S)[:, None], np.arange(S)[None, :]
    s = L.causal_scores(q.transpose(1, 0, 2), k.transpose(1, 0, 2), o["scale"])
    if o.get("distance_bias"):
        s = s - R.alibi_slopes(H)[:, None, None] * (i - j)
    if talk is not None:
        s = L.mix_heads(s, talk.astype(np.float64))
    s = np.where((j <= i) & (i - j < (o.get("window") or S)), s, -np.inf)
    top = s.max(-1, keepdims=True)
    if o.get("zero_sink"):
        top = np.maximum(top, 0.0)
    e = np.exp(s - top)
    return e / (e.sum(-1, keepdims=True) + (np.exp(-top) if o.get("zero_sink") else 0.0))


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


def turned(heads, kv_heads, dim, vdim, rot, window=0, **kw):
    """Rotated unit heads, mixed scores, a sink: what a Lufatar layer asks for."""
    o = dict(distance_bias=0, temp_every=0, rot_dims=rot, rot_base=1e4, unit_heads=1, mix_scores=1, zero_sink=1, norm_eps=1e-3)
    o.update(kw)
    return options(heads, kv_heads, dim, vdim, window, **o)


MIXED = {  # name: (options, batch, portions, norms, talk)
    "whole": (turned(4, 2, 16, 20, 8), 1, [40], False, True),
    "token_by_token": (turned(4, 4, 16, 20, 16), 2, [1] * 24, False, True),
    "twos_and_threes": (turned(6, 2, 12, 8, 4), 1, [2, 3, 2, 1, 3, 2, 9, 1], False, True),
    "odd_sizes": (turned(6, 2, 10, 7, 6), 1, [13, 2, 30, 1, 1, 9], False, True),
    "odd_value_size": (turned(6, 2, 12, 7, 6), 1, [13, 2, 30, 1, 1, 9], False, True),
    "one_head": (turned(1, 1, 8, 12, 2), 1, [20, 3, 1, 1], False, True),
    "three_heads": (turned(3, 1, 12, 20, 4), 2, [50, 2, 5, 1], False, True),
    "ten_per_kv_head": (turned(10, 1, 8, 8, 8), 1, [30, 1, 2], False, True),
    "many_heads": (turned(24, 4, 32, 16, 10), 1, [70, 1, 1, 20], False, True),
    "more_heads_than_tiles_take": (turned(40, 8, 8, 8, 8), 1, [30, 1, 10], False, True),
    "wide": (turned(4, 2, 128, 96, 64), 1, [64, 1, 33], False, True),
    "wider_than_tiles_take": (turned(2, 1, 160, 144, 150), 1, [30, 1, 12], False, True),
    "widest": (turned(2, 2, 300, 260, 20), 1, [11, 1, 2], False, True),
    "no_rotation": (turned(4, 2, 16, 16, 0), 1, [40, 1, 1, 10, 30], False, True),
    "not_unit": (turned(4, 2, 16, 16, 8, unit_heads=0), 1, [40, 1, 1, 10], False, True),
    "no_sink": (turned(4, 2, 16, 16, 8, zero_sink=0), 1, [40, 1, 1, 10], False, True),
    "mixed_behind_the_softmax": (turned(4, 2, 16, 16, 8, mix_scores=0), 1, [40, 1, 1, 10], False, True),
    "a_sink_alone": (options(8, 4, 16, 16, 0, distance_bias=0, temp_every=0, zero_sink=1), 1, [45, 1, 12], False, False),
    "a_sink_behind_norms": (options(8, 4, 16, 16, 21, zero_sink=1), 1, [45, 1, 12], True, True),
    "everything": (turned(8, 2, 32, 32, 16, window=21, distance_bias=1, temp_every=7), 1, [45, 1, 2, 12, 9], True, True),
    "norms": (turned(4, 2, 16, 16, 8), 1, [45, 1, 2, 12], True, True),
    "window_1": (turned(4, 2, 16, 16, 8, window=1), 1, [12, 1, 1, 4], False, True),
    "window_in_steps": (turned(4, 2, 16, 16, 8, window=11), 2, [30, 1, 1, 2, 1, 12], False, True),
    "segments_of_keys": (turned(4, 1, 16, 16, 16, rot_base=3e5), 1, [600, 1, 1, 5, 1], False, True),
    "long_prompt_then_decode": (turned(2, 1, 16, 16, 8, scale=2.0), 1, [700] + [1] * 12, False, True),
    "large_scores": (turned(4, 2, 16, 16, 8, scale=9.0), 1, [90, 1, 30, 2], False, True),
    "keys_cut_over_workgroups": (turned(16, 4, 64, 64, 32), 1, [640, 100, 1, 1], False, True),
    "eight_tokens": (turned(8, 2, 32, 24, 32), 3, [8, 8, 5, 8, 1], False, True),
}


def run_mixed_case(be, name):
    o, B, portions, norms, talk = MIXED[name]
    rng = np.random.default_rng(sum(map(ord, name)))
    check_attention(be, attention_case(rng, B, sum(portions), o, norms, talk), o, portions, tol=6e-5)


def run_mixed_needles(be, o, portions):
    """One key that stands out by far for one query, at every distance that matters: across portions, at segments' and key
    tiles' edges, at the first token, far back."""
    S, H, G, D = sum(portions), o["heads"], o["kv_heads"], o["dim"]
    o = {**o, "rot_dims": 0}
    rng = np.random.default_rng(S)
    ends = np.cumsum(portions)
    rows = sorted({int(i) for e in ends for i in (e - 1, e, e + 1) if 0 <= i < S})
    for i in rows:
        for j in sorted({0, 1, i, i - 1, i // 2, i - 15, i - 16, i - 17, i - 63, i - 64, i - 65, i - 128} & set(range(i + 1))):
            t = attention_case(rng, 1, S, o, norms=False)
            needle = rng.standard_normal(D)
            for n, heads, at in (("k", G, j), ("q", H, i)):
                t[n][0, at] = np.tile(needle, heads)
            t["talk"] = (np.eye(H) + 0.05).astype(np.float32)
            got = run_attention(be, t, o, portions)[0, i]
            want = attention_reference(t["q"][0], t["k"][0], t["v"][0], o, None, None, t["talk"])[i]
            close(got, want, 1e-4, f"row {i} looking at key {j}, portions {portions}")


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


# ---- embeddings of pairs ---------------------------------------------------------------------------------------------
def run_pair_embedding(be, dtype, B=2, vocab=37, buckets=13, width=20, mul_prev=1000003, mul_cur=8191, portions=(5, 1, 1, 2, 9)):
    rng = np.random.default_rng(buckets)
    table, pairs = bf16(rng.standard_normal((vocab, width))), bf16(rng.standard_normal((buckets + 1, width)))
    ids = rng.integers(0, vocab, size=(B, sum(portions)), dtype=np.uint32)
    want = np.stack([table[t].astype(np.float64) + pairs[L.bigram_rows(t, mul_prev, mul_cur, buckets)] for t in ids])
    wt, wp = weight(be, table, dtype), weight(be, pairs, dtype)
    prev, at = be.zeros((B, 0), 4), 0
    for n in portions:
        out, prev = be.block_pair_embedding({"ids": be.from_numpy(np.ascontiguousarray(ids[:, at:at + n])), "previous": prev, "table": wt, "pairs": wp},
                                            mul_prev=mul_prev, mul_cur=mul_cur)
        np.testing.assert_allclose(be.to_numpy(out), want[:, at:at + n], rtol=1e-6, atol=1e-6)
        at += n
        np.testing.assert_array_equal(be.to_numpy(prev), ids[:, at - 1:at])


# ---- grouped norms with filters --------------------------------------------------------------------------------------
CONV = [  # batch, portions, width, groups, taps, products, dtype
    (1, [30], 32, 4, 4, 2, "f32"), (2, [1] * 9, 32, 2, 4, 2, "f32"), (1, [2, 1, 2, 3, 9, 1, 40], 48, 3, 4, 2, "f32"), (1, [12, 2, 5], 30, 5, 3, 1, "f32"),
    (1, [12, 1, 5], 64, 1, 1, 2, "f32"), (2, [7, 2, 30], 64, 64, 2, 2, "f32"), (1, [3, 1, 2, 2, 40], 40, 2, 7, 2, "f32"), (1, [1, 1, 2, 40], 24, 2, 16, 1, "f32"),
    (1, [300, 1, 40], 520, 4, 4, 2, "bf16"), (3, [1, 1, 2, 90], 256, 4, 4, 2, "bf16"), (1, [20, 1, 9], 30, 2, 4, 2, "bf16"), (4, [600, 1], 128, 8, 4, 2, "bf16"),
    (1, [2000], 96, 4, 5, 2, "f32"), (1, [300], 1024, 4, 4, 2, "bf16")]


def run_conv_linear(be, case, seed=0):
    B, portions, W, groups, taps, n, dt = case
    rng = np.random.default_rng(seed)
    S, eps = sum(portions), 2e-3
    x = rng.standard_normal((B, S, W)).astype(np.float32) * (1 + np.arange(W, dtype=np.float32) / W)
    gam, conv = [(1 + 0.3 * rng.standard_normal(W)).astype(np.float32) for _ in range(n)], [rng.standard_normal((W, taps)).astype(np.float32) for _ in range(n)]
    w = [bf16(rng.standard_normal((N, W)) * W ** -0.5) for N in (50, 9)[:n]]
    want_h = [np.stack([L.with_causal_conv(L.group_norm(x[b].astype(np.float64), gam[i].astype(np.float64), groups, eps), conv[i].astype(np.float64))
                        for b in range(B)]) for i in range(n)]
    keep16 = dt == "bf16"
    wt = [weight(be, a, dt) for a in w]
    state, at = be.zeros((B, taps - 1, W), 0), 0
    for m in portions:
        ins = [{"gamma": be.from_numpy(gam[i]), "conv": be.from_numpy(conv[i]), "w": wt[i], "keep": i == n - 1, "keep_bf16": keep16} for i in range(n)]
        y, h, state = be.block_conv_linear(part_of_rows(be, x[:, at:at + m]), state, ins, groups=groups, eps=eps)
        tol = 2e-5 if dt == "f32" else 3e-2
        assert [k is None for k in h] == [i != n - 1 for i in range(n)]
        for i in range(n):
            close(be.to_numpy(y[i]), want_h[i][:, at:at + m] @ w[i].T.astype(np.float64), tol, f"product {i}, {case}, tokens {at} ..")
        close(be.to_numpy(be.cast(h[n - 1], 0)), want_h[n - 1][:, at:at + m], tol, f"kept rows, {case}")
        at += m
    z = L.rms(x.astype(np.float64).reshape(B, S, groups, -1), eps).reshape(B, S, W)
    z = np.concatenate([np.zeros((B, taps - 1, W)), z], 1)[:, S:]
    if taps > 1:
        close(be.to_numpy(state), z, 1e-5, f"state, {case}")


def run_grouped_linear(be, rows, K, groups, n, dt):
    rng = np.random.default_rng(rows)
    x, gamma, w = rng.standard_normal((1, rows, K)).astype(np.float32), (1 + 0.3 * rng.standard_normal(K)).astype(np.float32), bf16(rng.standard_normal((n, K)) * K ** -0.5)
    out = be.block_linear(part_of_rows(be, x), weight(be, w, dt), gamma=be.from_numpy(gamma), eps=1e-3, scale=0.7, groups=groups)
    want = L.group_norm(x[0].astype(np.float64), gamma.astype(np.float64), groups, 1e-3) @ w.T.astype(np.float64) * 0.7
    close(be.to_numpy(out)[0], want, 2e-5 if dt == "f32" else 1.5e-2, f"grouped linear {rows} {K} {groups}")


# ---- mixtures of experts ---------------------------------------------------------------------------------------------
EXPERTS = [  # rows, width, experts, top, groups, keep, ff, K of the branch (0: none), dtype
    (1, 32, 8, 2, 2, 1, 24, 40, "f32"), (1, 32, 8, 3, 4, 2, 24, 40, "bf16"), (4, 64, 16, 4, 4, 2, 48, 64, "f32"), (8, 520, 12, 3, 3, 2, 136, 264, "bf16"),
    (3, 30, 6, 2, 2, 1, 10, 14, "f32"), (3, 30, 6, 2, 2, 1, 10, 14, "bf16"), (1, 1024, 32, 8, 4, 2, 384, 1024, "bf16"), (4, 2048, 32, 8, 4, 2, 256, 512, "bf16"),
    (9, 32, 8, 2, 2, 1, 24, 40, "f32"), (40, 64, 16, 4, 4, 2, 48, 64, "f32"), (300, 128, 14, 3, 2, 1, 88, 128, "bf16"), (300, 128, 14, 3, 2, 1, 88, 128, "f32"),
    (70, 30, 6, 2, 2, 1, 10, 14, "f32"), (70, 30, 6, 2, 2, 1, 10, 14, "bf16"), (33, 64, 5, 5, 1, 1, 40, 0, "f32"), (2, 64, 5, 5, 1, 1, 40, 0, "f32"),
    (100, 64, 4, 1, 4, 1, 32, 48, "bf16"), (1, 64, 4, 1, 4, 1, 32, 48, "f32"), (2, 64, 4, 2, 4, 2, 32, 48, "f32"), (1, 64, 1, 1, 1, 1, 32, 48, "f32"),
    (50, 64, 1, 1, 1, 1, 32, 48, "f32"), (50, 72, 200, 6, 8, 3, 24, 48, "f32"), (2, 72, 200, 6, 8, 3, 24, 48, "f32"), (1100, 256, 8, 2, 2, 2, 200, 64, "bf16"),
    (700, 136, 8, 4, 2, 1, 72, 136, "f32"), (20, 2056, 4, 2, 2, 1, 40, 48, "bf16")]


def expert_case(rng, rows, width, count, ff, dt):
    h = rng.standard_normal((1, rows, width)).astype(np.float32)
    if dt == "bf16":
        h = bf16(h)
    return {"h": h, "logits": rng.standard_normal((1, rows, count)).astype(np.float32), "correction": rng.standard_normal(count).astype(np.float32),
            "gate_up": bf16(rng.standard_normal((count, 2, ff, width)) * 2.0 * width ** -0.5), "down": bf16(rng.standard_normal((count, width, ff)) * ff ** -0.5)}


def experts_reference(t, top, groups, keep, limit):
    h, z = t["h"][0].astype(np.float64), t["logits"][0].astype(np.float64)
    s, out = L.sigmoid(z), np.zeros(t["h"][0].shape)
    for r in range(len(h)):
        for e in L.chosen_experts(s[r] + t["correction"], top, groups, keep):
            out[r] += s[r, e] * L.expert(h[r], t["gate_up"][e, 0].astype(np.float64), t["gate_up"][e, 1].astype(np.float64), t["down"][e].astype(np.float64), limit)
    return out


def run_experts(be, case, seed=0, change=None):
    rows, width, count, top, groups, keep, ff, K, dt = case
    rng = np.random.default_rng(seed + rows)
    t = expert_case(rng, rows, width, count, ff, dt)
    if change:
        change(t)
    x, limit, scale = rng.standard_normal((1, rows, width)).astype(np.float32), 1.2, 0.4
    want, br = x[0].astype(np.float64), []
    if K:
        y, w = rng.standard_normal((1, rows, K)).astype(np.float32), bf16(rng.standard_normal((width, K)) * K ** -0.5)
        want = want + scale * (y[0].astype(np.float64) @ w.T)
        br = [{"y": part_of_rows(be, y), "w": weight(be, w, dt)}]
    want = want + scale * experts_reference(t, top, groups, keep, limit)
    ex = {n: be.from_numpy(t[n]) for n in ("logits", "correction")}
    ex["h"] = be.from_numpy(t["h"]) if dt == "f32" else be.cast(be.from_numpy(t["h"]), BF16)
    ex.update({n: weight(be, t[n], dt) for n in ("gate_up", "down")})
    out = be.block_residual(be.from_numpy(x), br, scale=scale, experts=ex, top=top, groups=groups, keep=keep, limit=limit, slope=1.702)
    close(be.to_numpy(out)[0], want, 3e-5 if dt == "f32" else 2e-2, f"experts {case}")


def run_expert_choices(be, rows):
    """Routing where it is easily wrong: negative choice scores, groups that win by their second member, one expert for all
    tokens, all tokens on the last expert, corrections that choose but do not weigh."""
    case = (rows, 48, 8, 2, 4, 2, 24, 0, "f32")

    def negative(t):
        t["correction"][:] = -5.0 - np.arange(8)

    def second_member(t):
        t["logits"][:] = -9.0
        t["correction"][:] = [0.9, -3.0, 0.5, 0.45, 0.4, 0.39, 0.95, -3.0]

    def one_for_all(t):
        t["correction"][:] = [9, 8, 0, 0, 0, 0, 0, 0]

    def last_for_all(t):
        t["correction"][:] = [0, 0, 0, 0, 0, 0, 8, 9]
        t["logits"][:, ::2] = -4.0

    def no_weight_from_corrections(t):
        t["correction"][:] = 100.0 * t["correction"]

    for change in (negative, second_member, one_for_all, last_for_all, no_weight_from_corrections):
        run_experts(be, case, change=change)


# ---- the tokens' own vectors -----------------------------------------------------------------------------------------
SIDE = [(1, 32, 8, "f32"), (1, 64, 24, "bf16"), (3, 30, 5, "f32"), (8, 520, 64, "bf16"), (40, 64, 16, "f32"), (300, 128, 24, "bf16"), (70, 30, 5, "bf16"),
        (2, 1024, 256, "bf16"), (1, 96, 1, "f32"), (600, 96, 16, "f32"), (1, 2048, 64, "f32"), (4, 2048, 64, "bf16"), (1, 40, 300, "f32")]


def run_side(be, case):
    rows, W, dim, dt = case
    rng = np.random.default_rng(rows)
    vocab, first, scale, eps = 23, 2 * dim, 0.6, 1e-3
    x, table = rng.standard_normal((1, rows, W)).astype(np.float32), bf16(rng.standard_normal((vocab, 4 * dim)))
    ids = rng.integers(0, vocab, size=(1, rows), dtype=np.uint32)
    gate, proj, norm = bf16(rng.standard_normal((dim, W)) * W ** -0.5), bf16(rng.standard_normal((W, dim)) * dim ** -0.5), (1 + 0.3 * rng.standard_normal(W)).astype(np.float32)
    out = be.block_token_side({"x": part_of_rows(be, x), "ids": be.from_numpy(ids), "table": weight(be, table, dt), "gate": weight(be, gate, dt), "proj": weight(be, proj, dt),
                               "norm": be.from_numpy(norm)}, first=first, eps=eps, scale=scale)
    W64 = {"p.side.gate": gate.astype(np.float64), "p.side.proj": proj.astype(np.float64), "p.side.norm": norm.astype(np.float64)}
    want = L.token_side(x[0].astype(np.float64), W64, "p", table[ids[0], first:first + dim].astype(np.float64), scale, eps)
    close(be.to_numpy(out)[0], want, 2e-5 if dt == "f32" else 2e-2, f"token side {case}")
