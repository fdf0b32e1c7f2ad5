"""What is checked on models of decoder blocks, of whichever design: the package's request steps, batches and greedy
generation against the design's whole-sequence statement.  `D` is a Design."""
import json
import os

import numpy as np


class Design:
    """configs: name -> config.json's dictionary; reference: the module with `logits(config, W, tokens)`; random_params:
    (config, seed, name, dtype) -> (tensor name, array) pairs."""

    def __init__(self, configs, reference, random_params, tolerance):
        self.configs, self.reference, self.random_params, self.tolerance = configs, reference, random_params, tolerance

    def logits(self, name, p, tokens):
        return self.reference.logits(self.configs[name], p, tokens)


def params_of(D, name, seed=0, bf16=True, dtype="float32"):
    """Weights as a dictionary; bf16: rounded to bfloat16, as a model file holds them."""
    from block_cases import bf16 as rounded

    p = dict(D.random_params(D.configs[name], seed, name, dtype))
    return {n: rounded(w) for n, w in p.items()} if bf16 else p


def load(D, session, name, seed=0, dtype="float32"):
    p = params_of(D, name, seed, dtype=dtype)
    session.clear_params()
    session.load_config(D.configs[name], dtype)
    for n, w in p.items():
        session.set_param(n, w)
    return p


def tokens_of(D, name, n, seed=1):
    return np.random.default_rng(seed).integers(0, D.configs[name]["vocab"], size=n)


def run(session, tokens, portions, request=1, end=True):
    """Logits [len(tokens), vocab] of a request in these portions."""
    at, out = 0, []
    for n in portions:
        out.append(session.step(request, tokens[at:at + n], range(n)))
        at += n
    assert at == len(tokens)
    if end:
        session.end(request)
    return np.concatenate(out)


def close(got, want, tol, what):
    """Per position: root mean square of the difference over the vocabulary, over the scale of all of them."""
    scale = np.sqrt(((want - want.mean(-1, keepdims=True)) ** 2).mean())
    d = got - want
    err = np.sqrt(((d - d.mean(-1, keepdims=True)) ** 2).mean(-1)) / scale
    assert err.max() <= tol, f"{what}: {err.max():.3g} of the logits' scale at position {int(err.argmax())}, allowed {tol:.3g}"


PORTIONS = {"whole": [50], "token_by_token": [1] * 50, "halves": [25, 25], "twos_and_threes": [2, 3] * 10, "prompt_then_decode": [38] + [1] * 12,
            "uneven": [17, 2, 1, 9, 1, 1, 16, 3], "sixteens": [16, 16, 16, 2]}


def check_portions(D, session, name, how, dtype="float32"):
    p = load(D, session, name, dtype=dtype)
    t = tokens_of(D, name, 50)
    close(run(session, t, PORTIONS[how]), D.logits(name, p, t), D.tolerance[dtype], f"{name}, {how}, {dtype}")


def check_one_token(D, session, name):
    p = load(D, session, name)
    for seed in range(3):
        t = tokens_of(D, name, 1, seed)
        close(run(session, t, [1]), D.logits(name, p, t), D.tolerance["float32"], f"{name}, one token")


def check_interleaved(D, session, name, dtype="float32"):
    """Requests of unequal length, a step of each in turn, ended and begun again under the same numbers."""
    p = load(D, session, name, dtype=dtype)
    rng = np.random.default_rng(3)
    for round_ in range(2):
        reqs = {r: tokens_of(D, name, n, seed=10 * round_ + r) for r, n in ((1, 44), (2, 7), (3, 29), (4, 1))}
        at, got = dict.fromkeys(reqs, 0), {r: [] for r in reqs}
        while at:
            for r in list(at):
                n = int(min(rng.integers(1, 12), len(reqs[r]) - at[r]))
                got[r].append(session.step(r, reqs[r][at[r]:at[r] + n], range(n)))
                at[r] += n
                if at[r] == len(reqs[r]):
                    session.end(r)
                    del at[r]
        assert session.requests_in_progress() == 0
        for r, t in reqs.items():
            close(np.concatenate(got[r]), D.logits(name, p, t), D.tolerance[dtype], f"{name}, request {r} among others")


def check_long_decode(D, session, name, n=150, dtype="float32"):
    p = load(D, session, name, dtype=dtype)
    t = tokens_of(D, name, n)
    close(run(session, t, [5] + [1] * (n - 5)), D.logits(name, p, t), D.tolerance[dtype], f"{name}, decoding from token 5 to {n}")


def greedy(D, name, p, prompt, steps):
    toks, out, gaps = list(prompt), [], []
    for _ in range(steps + 1):
        lg = D.logits(name, p, toks)[-1]
        top = np.sort(lg)
        out.append(int(lg.argmax()))
        gaps.append((top[-1] - top[-2]) / lg.std())
        toks.append(out[-1])
    return out, gaps


def check_generate(D, session, name, steps=12):
    """Two prompts of equal length as a batch through the generate loop; a prompt through request steps that ask for the
    next token; both against recomputing the whole sequence for every token."""
    p = load(D, session, name)
    prompts = np.stack([tokens_of(D, name, 21, seed=s) for s in (5, 6)])
    got, _ = session.generate(prompts, steps)
    for b in range(2):
        want, gaps = greedy(D, name, p, prompts[b], steps)
        same = [int(x) for x in got[:, b]]
        for i, (a, w) in enumerate(zip(same, want)):
            if a != w:
                assert gaps[i] < 1e-3, f"{name}: token {i} of sequence {b} is {a}, not {w}"
                break
        toks, nxt = prompts[b], []
        for _ in range(steps + 1):
            _, t = session.step(9, toks, (), want_next=True)
            nxt.append(t)
            toks = [t]
        session.end(9)
        assert nxt == same


def check_batch_logits(D, session, name):
    """The logits of a batch's prompts in one run against each alone."""
    p = load(D, session, name)
    prompts = np.stack([tokens_of(D, name, 23, seed=s) for s in (7, 8, 9)])
    _, lg = session.forward(prompts)
    for b in range(3):
        close(lg[b], D.logits(name, p, prompts[b]), D.tolerance["float32"], f"{name}, sequence {b} of a batch")
    rows = [4, 23 + 22, 2 * 23]
    _, picked = session.forward_rows(prompts, rows)
    np.testing.assert_allclose(picked, lg.reshape(-1, lg.shape[-1])[rows], rtol=1e-6, atol=1e-6)


def write_model(D, folder, name, seed=0, dtype="float32"):
    """A model folder as the package loads it; the weights."""
    import torch
    from safetensors.torch import save_file

    p = params_of(D, name, seed, dtype=dtype)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(D.configs[name], f)
    save_file({n: torch.from_numpy(np.ascontiguousarray(w)).to(torch.bfloat16) for n, w in p.items()}, os.path.join(folder, "model.safetensors"))
    return p
