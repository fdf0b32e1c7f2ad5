"""Lufatar model folders: the tensors a config.json asks for, random weights of those shapes, configurations for
benchmarks.  The model itself is catgrad_amd/host/lufatar.hpp."""
from __future__ import annotations

import numpy as np


def param_shapes(config: dict):
    """(name, shape) of every tensor of a model with this configuration."""
    w, vocab, taps, side = config["width"], config["vocab"], config["canon"]["taps"], config["token_side"]["dim"]
    out = [("embed", (vocab, w)), ("bigram", (config["embedding"]["bigram"]["buckets"] + 1, w))]
    if config.get("loop"):
        out.append(("loop.step", (config["loop"]["times"], w)))
    out.append(("side.embed", (vocab, side * len(config["layers"]))))
    for i, l in enumerate(config["layers"]):
        p, m, f = f"l{i}", l["mixer"], l.get("mlp")
        H, G, dim, vdim = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        out += [(f"{p}.norm1", (w,)), (f"{p}.canon1", (w, taps)), (f"{p}.mix.q", (H * dim, w)), (f"{p}.mix.k", (G * dim, w)),
                (f"{p}.mix.v", (G * vdim, w)), (f"{p}.mix.talk", (H, H)), (f"{p}.mix.o", (w, H * vdim))]
        if f:
            n, ff = f["router"]["experts"], f["expert"]["ff"]
            out += [(f"{p}.norm2", (w,)), (f"{p}.canon2", (w, taps)), (f"{p}.mlp.router", (n, w)), (f"{p}.mlp.correction", (n,))]
            for e in range(n):
                out += [(f"{p}.mlp.e{e}.gate", (ff, w)), (f"{p}.mlp.e{e}.up", (ff, w)), (f"{p}.mlp.e{e}.down", (w, ff))]
        out += [(f"{p}.side.gate", (side, w)), (f"{p}.side.proj", (w, side)), (f"{p}.side.norm", (w,))]
    return out + [("final.norm", (w,)), ("head", (vocab, w))]


def random_params(config: dict, seed: int = 0):
    """Random weights, drawn in `param_shapes()` order: yields (name, float32 array).  Matrices keep their input's scale,
    norm weights scatter around one, head mixing around the identity.  Large expert matrices are cuts of one pool of draws."""
    rng = np.random.default_rng(seed)
    pool = None
    for name, shape in param_shapes(config):
        n = int(np.prod(shape))
        if ".mlp.e" in name and n >= 1 << 18:
            if pool is None or pool.size < 8 * n:
                pool = rng.standard_normal(8 * n, dtype=np.float32)
            at = int(rng.integers(0, pool.size - n + 1))
            yield name, (pool[at:at + n] * np.float32(shape[1] ** -0.5)).reshape(shape)
            continue
        x = rng.standard_normal(shape, dtype=np.float32)
        if name.endswith(("norm", "norm1", "norm2")):
            yield name, 1.0 + np.float32(0.2) * x
        elif name.endswith(".talk"):
            yield name, np.eye(shape[0], dtype=np.float32) + np.float32(0.3) * x
        elif name.endswith((".canon1", ".canon2")):
            yield name, x * np.float32(0.5 * shape[1] ** -0.5)
        elif name in ("embed", "bigram", "side.embed"):
            yield name, x
        elif name.endswith(".correction") or name == "loop.step":
            yield name, np.float32(0.2) * x
        else:
            x *= np.float32(shape[1] ** -0.5)
            yield name, x


def config_of(layers, vocab, width, loop=None, eps=1e-6, groups=4, mult=0.5, taps=4, side=16, buckets=61, mul_prev=31, mul_cur=7) -> dict:
    return {"architecture": "Lufatar", "layers": layers, "loop": loop, "norm": {"eps": eps, "groups": groups}, "residual_mult": mult,
            "canon": {"taps": taps}, "token_side": {"dim": side},
            "embedding": {"bigram": {"buckets": buckets, "mul_prev": mul_prev, "mul_cur": mul_cur}}, "vocab": vocab, "width": width}


def experts(count, top, ff, groups=1, keep=1, limit=1.5) -> dict:
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit},
            "router": {"experts": count, "top": top, "groups": {"count": groups, "keep": keep}}}


def attention_layer(heads, kv_heads, dim, vdim, mlp=None, rot=None, base=10000.0, scale=None) -> dict:
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                      "rot": {"dims": dim if rot is None else rot, "base": base}, "scale": dim ** -0.5 if scale is None else scale}}
