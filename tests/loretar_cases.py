"""Small Loretar models shared by the CPU and GPU tests, and what is checked on them: the package's request steps, batches
and greedy generation against the whole-sequence statement in loretar_reference.py."""
import numpy as np

import loretar_reference as R
from catgrad_amd.loretar import attention_layer, config_of, delta_layer, random_params


def layers_mixed():
    return [attention_layer(4, 2, 16, 16, 9, 40, coef=0.4, every=5), delta_layer(4, 2, 16, 24, 48, conv=4),
            attention_layer(6, 3, 8, 12, 14, 0, scale=0.5, coef=0.2, every=3), delta_layer(2, 2, 24, 16, 0, conv=3)]


CONFIGS = {
    "mixed": config_of(layers_mixed(), 71, 64, loop={"start": 1, "stop": 3, "times": 2}, eps=1e-4, logit_scale=0.7),
    "no_loop": config_of(layers_mixed(), 64, 32, eps=1e-5),
    "everything_looped": config_of(layers_mixed()[:3], 50, 48, loop={"start": 0, "stop": 3, "times": 3}, logit_scale=1.3),
    "a_loop_of_one_pass": config_of(layers_mixed()[:2], 50, 48, loop={"start": 1, "stop": 2, "times": 1}),
    "looped_to_the_end": config_of(layers_mixed(), 50, 40, loop={"start": 2, "stop": 4, "times": 2}),
    "odd_sizes": config_of([delta_layer(3, 1, 10, 7, 33, conv=2), attention_layer(3, 1, 10, 6, 7, 29, coef=0.3, every=2)], 37, 36,
                           loop={"start": 0, "stop": 1, "times": 2}),
    "one_head_each": config_of([attention_layer(1, 1, 12, 20, 5, 24), delta_layer(1, 1, 12, 20, 24, conv=1)], 41, 24),
    "a_window_of_one": config_of([attention_layer(4, 4, 8, 8, 1, 20), delta_layer(2, 1, 8, 8, 20)], 41, 32),
    "recurrence_only": config_of([delta_layer(4, 4, 16, 16, 40), delta_layer(4, 2, 32, 16, 0)], 64, 32, loop={"start": 0, "stop": 2, "times": 2}),
    "attention_only": config_of([attention_layer(8, 2, 16, 16, 20, 40), attention_layer(2, 1, 32, 8, 11, 0)], 64, 32),
    "wider": config_of([attention_layer(8, 4, 32, 48, 40, 320, every=20), delta_layer(4, 4, 48, 64, 256)], 300, 192,
                       loop={"start": 0, "stop": 2, "times": 2}),
}


def params_of(name, seed=0, bf16=True):
    """Weights as a dictionary; bf16: rounded to bfloat16, as a model file holds them."""
    from block_cases import bf16 as rounded

    p = dict(random_params(CONFIGS[name], seed, low_rank=5 if name == "odd_sizes" else 8))
    return {n: rounded(w) for n, w in p.items()} if bf16 else p


def load(session, name, seed=0, dtype="float32"):
    p = params_of(name, seed)
    session.clear_params()
    session.load_config(CONFIGS[name], dtype)
    for n, w in p.items():
        session.set_param(n, w)
    return p


def tokens_of(name, n, seed=1):
    return np.random.default_rng(seed).integers(0, CONFIGS[name]["vocab"], size=n)


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


TOLERANCE = {"float32": 5e-5, "bfloat16": 4e-2}
PORTIONS = {"whole": [50], "token_by_token": [1] * 50, "halves": [25, 25], "twos_and_threes": [2, 3] * 10, "prompt_then_decode": [38] + [1] * 12,
            "uneven": [17, 2, 1, 9, 1, 1, 16, 3], "sixteens": [16, 16, 16, 2]}


def check_portions(session, name, how, dtype="float32"):
    p = load(session, name, dtype=dtype)
    t = tokens_of(name, 50)
    close(run(session, t, PORTIONS[how]), R.logits(CONFIGS[name], p, t), TOLERANCE[dtype], f"{name}, {how}, {dtype}")


def check_one_token(session, name):
    p = load(session, name)
    for seed in range(3):
        t = tokens_of(name, 1, seed)
        close(run(session, t, [1]), R.logits(CONFIGS[name], p, t), TOLERANCE["float32"], f"{name}, one token")


def check_interleaved(session, name, dtype="float32"):
    """Requests of unequal length, a step of each in turn, ended and begun again under the same numbers."""
    p = load(session, name, dtype=dtype)
    rng = np.random.default_rng(3)
    for round_ in range(2):
        reqs = {r: tokens_of(name, n, seed=10 * round_ + r) for r, n in ((1, 44), (2, 7), (3, 29), (4, 1))}
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
            close(np.concatenate(got[r]), R.logits(CONFIGS[name], p, t), TOLERANCE[dtype], f"{name}, request {r} among others")


def check_long_decode(session, name, n=150, dtype="float32"):
    p = load(session, name, dtype=dtype)
    t = tokens_of(name, n)
    close(run(session, t, [5] + [1] * (n - 5)), R.logits(CONFIGS[name], p, t), TOLERANCE[dtype], f"{name}, decoding from token 5 to {n}")


def greedy(config, p, prompt, steps):
    toks, out, gaps = list(prompt), [], []
    for _ in range(steps + 1):
        lg = R.logits(config, p, toks)[-1]
        top = np.sort(lg)
        out.append(int(lg.argmax()))
        gaps.append((top[-1] - top[-2]) / lg.std())
        toks.append(out[-1])
    return out, gaps


def check_generate(session, name, steps=12):
    """Two prompts of equal length as a batch through the generate loop; a prompt through request steps that ask for the
    next token; both against recomputing the whole sequence for every token."""
    p = load(session, name)
    prompts = np.stack([tokens_of(name, 21, seed=s) for s in (5, 6)])
    got, _ = session.generate(prompts, steps)
    for b in range(2):
        want, gaps = greedy(CONFIGS[name], p, prompts[b], steps)
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


def check_batch_logits(session, name):
    """The logits of a batch's prompts in one run against each alone."""
    p = load(session, name)
    prompts = np.stack([tokens_of(name, 23, seed=s) for s in (7, 8, 9)])
    _, lg = session.forward(prompts)
    for b in range(3):
        close(lg[b], R.logits(CONFIGS[name], p, prompts[b]), TOLERANCE["float32"], f"{name}, sequence {b} of a batch")
    rows = [4, 23 + 22, 2 * 23]
    _, picked = session.forward_rows(prompts, rows)
    np.testing.assert_allclose(picked, lg.reshape(-1, lg.shape[-1])[rows], rtol=1e-6, atol=1e-6)
