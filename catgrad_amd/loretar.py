"""Loretar model folders: the tensors a config.json asks for, random weights of those shapes, configurations for
benchmarks.  The model itself is catgrad_amd/host/loretar.hpp."""
from __future__ import annotations

import numpy as np


def param_shapes(config: dict, low_rank: int = 0):
    """(name, shape) of every tensor of a model with this configuration.  `low_rank`: inner size of the two factored
    projections of a channel_delta mixer, which only their tensors' shapes say (0: the mixer's vdim)."""
    w = config["width"]
    out = [("embed", (config["vocab"], w))]
    if config.get("loop"):
        out += [("loop.in", (w, 2 * w)), ("loop.step", (config["loop"]["times"], w))]
    for i, l in enumerate(config["layers"]):
        p, m = f"l{i}", l["mixer"]
        x = f"{p}.mix"
        H, G, dim, vdim = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        out.append((f"{p}.norm1", (w,)))
        if l["type"] == "attention":
            out += [(f"{x}.q", (H * dim, w)), (f"{x}.k", (G * dim, w)), (f"{x}.v", (G * vdim, w)), (f"{x}.q.norm", (H * dim,)),
                    (f"{x}.k.norm", (G * dim,)), (f"{x}.talk", (H, H))]
        else:
            r, taps = low_rank or vdim, m["conv"]
            out += [(f"{x}.q", (G * dim, w)), (f"{x}.q.conv", (G * dim, taps)), (f"{x}.k", (G * dim, w)), (f"{x}.k.conv", (G * dim, taps)),
                    (f"{x}.v", (H * vdim, w)), (f"{x}.v.conv", (H * vdim, taps)), (f"{x}.b", (H, w)), (f"{x}.A_log", (H,)),
                    (f"{x}.norm", (vdim,)), (f"{x}.a1", (r, w)), (f"{x}.a2", (H * dim, r)), (f"{x}.dt_bias", (H * dim,)),
                    (f"{x}.g1", (r, w)), (f"{x}.g2", (H * vdim, r))]
        out.append((f"{x}.o", (w, H * vdim)))
        if l.get("mlp"):
            ff = l["mlp"]["ff"]
            out += [(f"{p}.mlp.up", (ff, w)), (f"{p}.mlp.down", (w, ff)), (f"{p}.mlp.act", (4,))]
        for g in ("rg1", "rg2") if l.get("mlp") else ("rg1",):
            out += [(f"{p}.{g}", (w, w)), (f"{p}.{g}.b", (w,))]
    return out + [("final.norm", (w,)), ("head", (config["vocab"], w))]


def random_params(config: dict, seed: int = 0, low_rank: int = 0):
    """Random weights, drawn in `param_shapes()` order: yields (name, float32 array).  Matrices keep their input's scale,
    norm weights scatter around one, head mixing around the identity, decays between fast and slow."""
    rng = np.random.default_rng(seed)
    for name, shape in param_shapes(config, low_rank):
        n = rng.standard_normal(shape, dtype=np.float32)
        if name.endswith("norm") or name.endswith("norm1"):
            yield name, 1.0 + np.float32(0.2) * n
        elif name.endswith(".talk"):
            yield name, np.eye(shape[0], dtype=np.float32) + np.float32(0.3) * n
        elif name.endswith(".A_log"):
            yield name, np.float32(0.5) * n
        elif name.endswith(".dt_bias"):
            yield name, n - np.float32(3.0)
        elif name.endswith(".mlp.act"):
            yield name, np.float32(0.5) + np.float32(0.2) * n
        elif name.endswith(".conv"):
            yield name, n * np.float32(shape[1] ** -0.5)
        elif name == "embed":
            yield name, n
        elif len(shape) == 2 and name != "loop.step":
            n *= np.float32(shape[1] ** -0.5)
            yield name, n
        else:
            yield name, np.float32(0.2) * n


def config_of(layers, vocab, width, loop=None, eps=1e-6, logit_scale=1.0) -> dict:
    return {"architecture": "Loretar", "layers": layers, "loop": loop, "norm": {"eps": eps}, "logit_scale": logit_scale,
            "vocab": vocab, "width": width}


def attention_layer(heads, kv_heads, dim, vdim, window, ff, scale=None, coef=0.1, every=1024) -> dict:
    return {"type": "attention", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": window},
                      "q_temp": {"coef": coef, "every": every}, "scale": dim ** -0.5 if scale is None else scale}}


def delta_layer(heads, kv_heads, dim, vdim, ff, conv=4) -> dict:
    return {"type": "channel_delta", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}
