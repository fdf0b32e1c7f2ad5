"""A plain float64 statement of the Loretar decoder, one function per mechanism, for one sequence at a time.

Everything is written over whole sequences (no cache, no portions, no fused steps): attention scores every pair of
positions, the recurrence walks token by token.  It shares no code with the package; the tests compare the package with it.
`config` is the dictionary of a model's config.json, `W` a dictionary of float arrays named as in its weight file."""
import numpy as np


def sigmoid(x):
    return 0.5 * (1.0 + np.tanh(0.5 * x))


def silu(x):
    return x * sigmoid(x)


def softplus(x):
    return np.logaddexp(0.0, x)


def rms(x, eps):
    """x at a mean square of one along the last axis."""
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def rms_norm(x, w, eps):
    return rms(x, eps) * w


def poly_norm(z, coef, eps):
    a, b, c, e = coef
    return a * rms(z, eps) + b * rms(z ** 2, eps) + c * rms(z ** 3, eps) + e


def query_temperature(positions, coef, every):
    return 1.0 + coef * np.log(np.floor((positions + 1) / every) + 1.0)


def alibi_slopes(heads):
    return 2.0 ** (-8.0 * (np.arange(heads) + 1) / heads)


def attention_weights(q, k, scale, slopes, window):
    """q [H, S, dim], k [G, S, dim] -> soft-max weights [H, S, S]; window None: every earlier position is visible."""
    H, S, _ = q.shape
    rep = H // k.shape[0]
    i, j = np.arange(S)[:, None], np.arange(S)[None, :]
    visible = j <= i
    if window is not None:
        visible = visible & (i - j < window)
    out = np.zeros((H, S, S))
    for h in range(H):
        s = q[h] @ k[h // rep].T * scale
        if slopes is not None:
            s = s - slopes[h] * (i - j)
        s = np.where(visible, s, -np.inf)
        e = np.exp(s - s.max(-1, keepdims=True))
        out[h] = e / e.sum(-1, keepdims=True)
    return out


def attention_mixer(h, W, p, m, eps):
    S = h.shape[0]
    H, G, dim, vdim = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm(h @ W[p + ".q"].T, W[p + ".q.norm"], eps)
    k = rms_norm(h @ W[p + ".k"].T, W[p + ".k.norm"], eps)
    v = h @ W[p + ".v"].T
    t = m["q_temp"]
    q = q * query_temperature(np.arange(S), t["coef"], t["every"])[:, None]
    q = q.reshape(S, H, dim).transpose(1, 0, 2)
    k = k.reshape(S, G, dim).transpose(1, 0, 2)
    v = v.reshape(S, G, vdim).transpose(1, 0, 2)
    w = attention_weights(q, k, m["scale"], alibi_slopes(H), m["mask"]["size"])
    w = np.tensordot(W[p + ".talk"], w, axes=(1, 0))
    o = np.stack([w[i] @ v[i // (H // G)] for i in range(H)], 1)
    return o.reshape(S, H * vdim) @ W[p + ".o"].T


def short_conv(x, taps):
    """Causal convolution per channel: x [S, C], taps [C, n] in time order."""
    S, C = x.shape
    n = taps.shape[1]
    padded = np.concatenate([np.zeros((n - 1, C)), x])
    return sum(padded[t:t + S] * taps[:, t] for t in range(n))


def unit(x):
    return x / np.sqrt((x * x).sum(-1, keepdims=True) + 1e-6)


def channel_decay(a, A_log, dt_bias, heads, dim):
    """a [S, heads * dim] -> the factor on every key channel's row of the state, [S, heads, dim]."""
    s = softplus(a + dt_bias).reshape(-1, heads, dim)
    return np.exp(-np.exp(A_log)[None, :, None] * s)


def delta_rule(q, k, v, beta, g, S0=None):
    """q, k [S, H, dim], v [S, H, vdim], beta [S, H], g [S, H, dim] -> (o [S, H, vdim], final state [H, dim, vdim])."""
    T, H, dim = q.shape
    st = np.zeros((H, dim, v.shape[2])) if S0 is None else S0.copy()
    o = np.zeros(v.shape)
    for t in range(T):
        for h in range(H):
            s = g[t, h][:, None] * st[h]
            u = beta[t, h] * (v[t, h] - s.T @ k[t, h])
            s = s + np.outer(k[t, h], u)
            o[t, h] = s.T @ q[t, h]
            st[h] = s
    return o, st


def channel_delta_mixer(h, W, p, m, eps):
    S = h.shape[0]
    H, G, dim, vdim = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    rep = H // G
    q = silu(short_conv(h @ W[p + ".q"].T, W[p + ".q.conv"])).reshape(S, G, dim)
    k = silu(short_conv(h @ W[p + ".k"].T, W[p + ".k.conv"])).reshape(S, G, dim)
    v = silu(short_conv(h @ W[p + ".v"].T, W[p + ".v.conv"])).reshape(S, H, vdim)
    q, k = unit(q) * dim ** -0.5, unit(k)
    q, k = np.repeat(q, rep, 1), np.repeat(k, rep, 1)
    beta = sigmoid(h @ W[p + ".b"].T)
    g = channel_decay((h @ W[p + ".a1"].T) @ W[p + ".a2"].T, W[p + ".A_log"], W[p + ".dt_bias"], H, dim)
    o, _ = delta_rule(q, k, v, beta, g)
    gate = sigmoid((h @ W[p + ".g1"].T) @ W[p + ".g2"].T).reshape(S, H, vdim)
    o = rms_norm(o, W[p + ".norm"], eps) * gate
    return o.reshape(S, H * vdim) @ W[p + ".o"].T


MIXERS = {"attention": attention_mixer, "channel_delta": channel_delta_mixer}


def gate(h, W, b):
    return sigmoid(h @ W.T + b)


def layer(x, W, p, spec, eps):
    h = rms_norm(x, W[p + ".norm1"], eps)
    y = MIXERS[spec["type"]](h, W, p + ".mix", spec["mixer"], eps) * gate(h, W[p + ".rg1"], W[p + ".rg1.b"])
    if spec.get("mlp"):
        f = poly_norm(h @ W[p + ".mlp.up"].T, W[p + ".mlp.act"], eps) @ W[p + ".mlp.down"].T
        y = y + f * gate(h, W[p + ".rg2"], W[p + ".rg2.b"])
    return x + y


def run_order(config):
    """(layer, first of which pass or None) in the order of evaluation."""
    n = len(config["layers"])
    lp = config.get("loop")
    if not lp:
        return [(i, None) for i in range(n)]
    out = [(i, None) for i in range(lp["start"])]
    for t in range(lp["times"]):
        out += [(i, t if i == lp["start"] else None) for i in range(lp["start"], lp["stop"])]
    return out + [(i, None) for i in range(lp["stop"], n)]


def hidden_states(config, W, tokens):
    """Residual stream after every layer run: a list of [S, width]."""
    W = {k: np.asarray(v, dtype=np.float64) for k, v in W.items()}
    eps = config["norm"]["eps"]
    x0 = W["embed"][np.asarray(tokens)]
    x, out = x0, []
    for i, begins in run_order(config):
        if begins is not None:
            x = np.concatenate([x, x0], -1) @ W["loop.in"].T + W["loop.step"][begins]
        x = layer(x, W, f"l{i}", config["layers"][i], eps)
        out.append(x)
    return out


def logits(config, W, tokens):
    x = hidden_states(config, W, tokens)[-1]
    W = {k: np.asarray(W[k], dtype=np.float64) for k in ("final.norm", "head")}
    return rms_norm(x, W["final.norm"], config["norm"]["eps"]) @ W["head"].T * config["logit_scale"]
