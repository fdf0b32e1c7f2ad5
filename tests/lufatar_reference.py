"""A plain float64 statement of the Lufatar decoder, one function per mechanism, for one sequence at a time.

Everything is written over whole sequences (no cache, no portions, no fused steps).  It shares no code with the package;
the tests compare the package with it.  `config` is the dictionary of a model's config.json, `W` a dictionary of float
arrays named as in its weight file."""
import numpy as np


def sigmoid(x):
    return 0.5 * (1.0 + np.tanh(0.5 * x))


def gelu_tanh(x):
    return 0.5 * x * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (x + 0.044715 * x ** 3)))


def rms(x, eps):
    """x at a mean square of one along the last axis."""
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def group_norm(x, w, groups, eps):
    """Every one of `groups` equal runs of x's last axis at a mean square of one, then times w."""
    parts = x.reshape(x.shape[:-1] + (groups, -1))
    return rms(parts, eps).reshape(x.shape) * w


def bigram_rows(tokens, mul_prev, mul_cur, buckets):
    """The row of the bigram table for every token; the row behind the buckets for a token that follows none."""
    out = [buckets]
    for a, b in zip(tokens[:-1], tokens[1:]):
        out.append((int(a) * mul_prev + int(b) * mul_cur) % buckets)
    return np.array(out[:len(tokens)])


def embedding(W, config, tokens):
    g = config["embedding"]["bigram"]
    tokens = np.asarray(tokens)
    return W["embed"][tokens] + W["bigram"][bigram_rows(tokens, g["mul_prev"], g["mul_cur"], g["buckets"])]


def with_causal_conv(h, taps):
    """h plus its causal convolution over time, channel by channel: h [S, C], taps [C, n] in time order."""
    S, C = h.shape
    n = taps.shape[1]
    padded = np.concatenate([np.zeros((n - 1, C)), h])
    return h + sum(padded[t:t + S] * taps[:, t] for t in range(n))


def rotate_pairs(x, positions, base, dims):
    """x [S, heads, dim]: the first `dims` values of a head as pairs of neighbours, each turned by position * base^(-2 i / dims)."""
    out = x.copy()
    if not dims:
        return out
    a = positions[:, None] * base ** (-2.0 * np.arange(dims // 2) / dims)
    c, s = np.cos(a)[:, None, :], np.sin(a)[:, None, :]
    u, v = x[:, :, 0:dims:2], x[:, :, 1:dims:2]
    out[:, :, 0:dims:2], out[:, :, 1:dims:2] = u * c - v * s, v * c + u * s
    return out


def causal_scores(q, k, scale):
    """q [S, H, dim], k [S, G, dim] -> [H, S, S]; a group of query heads shares a key head."""
    S, H, _ = q.shape
    rep = H // k.shape[1]
    return np.stack([q[:, h] @ k[:, h // rep].T * scale for h in range(H)])


def mix_heads(scores, T):
    return np.tensordot(T, scores, axes=(1, 0))


def softmax_beside_zero(scores):
    """Causal soft-max over the last axis with another score of 0 in the sum, whose weight goes nowhere."""
    S = scores.shape[-1]
    s = np.where(np.arange(S)[None, :] <= np.arange(S)[:, None], scores, -np.inf)
    top = np.maximum(s.max(-1, keepdims=True), 0.0)
    e = np.exp(s - top)
    return e / (np.exp(-top) + e.sum(-1, keepdims=True))


def attention_mixer(h, W, p, m, eps):
    S = h.shape[0]
    H, G, dim, vdim = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos = np.arange(S)
    turn = lambda x: rms(rotate_pairs(x, pos, m["rot"]["base"], m["rot"]["dims"]), eps)
    q = turn((h @ W[p + ".q"].T).reshape(S, H, dim))
    k = turn((h @ W[p + ".k"].T).reshape(S, G, dim))
    v = (h @ W[p + ".v"].T).reshape(S, G, vdim)
    w = softmax_beside_zero(mix_heads(causal_scores(q, k, m["scale"]), W[p + ".talk"]))
    o = np.stack([w[i] @ v[:, i // (H // G)] for i in range(H)], 1)
    return o.reshape(S, H * vdim) @ W[p + ".o"].T


MIXERS = {"attention": attention_mixer}


def chosen_experts(choice, top, groups, keep):
    """choice [experts] -> the numbers of the chosen ones: only members of the `keep` best groups, a group being as good as
    the sum of its two best members, and of those the `top` best."""
    size = len(choice) // groups
    by_group = choice.reshape(groups, size)
    worth = np.sort(by_group, -1)[:, -2:].sum(-1)
    best = np.argsort(-worth, kind="stable")[:keep]
    allowed = np.full(len(choice), -np.inf)
    for g in best:
        allowed[g * size:(g + 1) * size] = by_group[g]
    return np.argsort(-allowed, kind="stable")[:top]


def expert(h, gate, up, down, limit):
    g = np.minimum(h @ gate.T, limit)
    u = np.clip(h @ up.T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ down.T


def moe(h, W, p, spec):
    r = spec["router"]
    groups = r.get("groups") or {"count": 1, "keep": 1}
    s = sigmoid(h @ W[p + ".router"].T)
    out = np.zeros_like(h)
    for t in range(len(h)):
        for e in chosen_experts(s[t] + W[p + ".correction"], r["top"], groups["count"], groups["keep"]):
            q = f"{p}.e{e}"
            out[t] += s[t, e] * expert(h[t], W[q + ".gate"], W[q + ".up"], W[q + ".down"], spec["expert"]["limit"])
    return out


def token_side(x, W, p, e, mult, eps):
    """x and what its token's own vector e, gated by x, adds to it."""
    y = (gelu_tanh(x @ W[p + ".side.gate"].T) * e) @ W[p + ".side.proj"].T
    return x + mult * rms(y, eps) * W[p + ".side.norm"]


def layer(x, W, p, spec, config, e):
    eps, groups, m = config["norm"]["eps"], config["norm"]["groups"], config["residual_mult"]
    h = with_causal_conv(group_norm(x, W[p + ".norm1"], groups, eps), W[p + ".canon1"])
    y = MIXERS[spec["type"]](h, W, p + ".mix", spec["mixer"], eps)
    if spec.get("mlp"):
        h = with_causal_conv(group_norm(x, W[p + ".norm2"], groups, eps), W[p + ".canon2"])
        y = y + moe(h, W, p + ".mlp", spec["mlp"])
    return token_side(x + m * y, W, p, e, m, eps)


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
    d = config["token_side"]["dim"]
    side = W["side.embed"][np.asarray(tokens)]
    x, out = embedding(W, config, tokens), []
    for i, begins in run_order(config):
        if begins is not None:
            x = x + W["loop.step"][begins]
        x = layer(x, W, f"l{i}", config["layers"][i], config, side[:, i * d:(i + 1) * d])
        out.append(x)
    return out


def logits(config, W, tokens):
    x = hidden_states(config, W, tokens)[-1]
    W = {k: np.asarray(W[k], dtype=np.float64) for k in ("final.norm", "head")}
    return group_norm(x, W["final.norm"], config["norm"]["groups"], config["norm"]["eps"]) @ W["head"].T
