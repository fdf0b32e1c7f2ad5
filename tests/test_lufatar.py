"""The Lufatar model of the host driver on the CPU oracle: configuration, weights, request states, generation and the trace
runner against the plain statement in lufatar_reference.py."""
import copy
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import design_cases as C
import lufatar_reference as R
from lufatar_cases import LUFATAR as D
from catgrad_amd.lufatar import param_shapes
from catgrad_amd.runner import Session
from oracle_loader import ORACLE_LIB, oracle_library

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


@pytest.fixture(scope="module")
def session():
    oracle_library()
    return Session(ORACLE_LIB)


@pytest.mark.parametrize("name", list(D.configs))
def test_whole_prompt(session, name):
    C.check_portions(D, session, name, "whole")


@pytest.mark.parametrize("how", [h for h in C.PORTIONS if h != "whole"])
@pytest.mark.parametrize("name", ["mixed", "odd_sizes", "one_of_each"])
def test_portions(session, name, how):
    C.check_portions(D, session, name, how)


@pytest.mark.parametrize("name", ["mixed", "no_loop", "everything_looped"])
def test_bfloat16_weights(session, name):
    C.check_portions(D, session, name, "prompt_then_decode", "bfloat16")


def test_one_token(session):
    C.check_one_token(D, session, "mixed")


def test_interleaved_requests(session):
    C.check_interleaved(D, session, "mixed")


def test_long_decode(session):
    C.check_long_decode(D, session, "no_loop")


@pytest.mark.parametrize("name", ["mixed", "attention_only"])
def test_generate(session, name):
    C.check_generate(D, session, name, steps=6)


def test_batch_logits(session):
    C.check_batch_logits(D, session, "mixed")


def test_recorded_schedules(session):
    """The layered and the recorded evaluation orders run the same operations."""
    C.load(D, session, "mixed")
    t = C.tokens_of(D, "mixed", 30)
    want = C.run(session, t, [20, 1, 9])
    try:
        for schedule in (1, 2):
            session.set_schedule(schedule)
            np.testing.assert_array_equal(C.run(session, t, [20, 1, 9]), want)
    finally:
        session.set_schedule(0)


def test_a_parameter_set_again_is_used(session):
    p = C.load(D, session, "mixed")
    t = C.tokens_of(D, "mixed", 12)
    C.run(session, t, [12])
    p["l1.mix.k"] = p["l1.mix.k"] * np.float32(-0.5)
    session.set_param("l1.mix.k", p["l1.mix.k"])
    C.close(C.run(session, t, [12]), R.logits(D.configs["mixed"], p, t), 5e-5, "after a parameter was set again")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_model_folder(session, tmp_path, dtype):
    p = C.write_model(D, tmp_path, "everything_looped", dtype=dtype)
    stats = session.load_pretrained(tmp_path, dtype)
    assert stats["tensors"] == len(p)
    t = C.tokens_of(D, "everything_looped", 30)
    C.close(C.run(session, t, [20, 1, 9]), R.logits(D.configs["everything_looped"], p, t), D.tolerance[dtype], f"model folder, {dtype}")


def test_trace_run(tmp_path):
    """Two requests step by step through the program: wanted places, steps without any, ends, and a name used again."""
    model, out = tmp_path / "model", tmp_path / "out"
    model.mkdir(), out.mkdir()
    p = C.write_model(D, model, "mixed")
    c = D.configs["mixed"]
    a, b = C.tokens_of(D, "mixed", 26, 1), C.tokens_of(D, "mixed", 9, 2)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": a[:20].tolist(), "want": [0, 19]}], "end": []},
             {"step": 1, "entries": [{"id": "y", "tokens": b[:7].tolist(), "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": a[20:].tolist(), "want": [5, 2]}], "end": ["x"]},
             {"step": 3, "entries": [{"id": "x", "tokens": b.tolist(), "want": [8]}], "end": []},
             {"step": 5, "entries": [{"id": "y", "tokens": b[7:].tolist(), "want": [1]}, {"id": "x", "tokens": [3], "want": [0]}], "end": ["x", "y"]}]
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", str(model), "--dtype", "float32", "--out", str(out),
                        "--max-tokens", "64", "--backend-library", ORACLE_LIB], input="".join(json.dumps(s) + "\n" for s in steps), text=True,
                       stdout=subprocess.PIPE, timeout=120)
    assert r.returncode == 0
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == [f"done {s['step']}" for s in steps]
    assert sorted(os.listdir(out)) == ["0.f32", "2.f32", "3.f32", "5.f32"]
    la, lb = R.logits(c, p, a), R.logits(c, p, list(b) + [3])
    for step, want in ((0, la[[0, 19]]), (2, la[[25, 22]]), (3, lb[[8]]), (5, lb[[8, 9]])):
        got = np.fromfile(out / f"{step}.f32", "<f4").reshape(len(want), c["vocab"])
        C.close(got, want, 5e-5, f"step {step}")
    bad = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", "float32", "--out", str(out),
                          "--max-tokens", "64", "--backend-library", ORACLE_LIB], input="", text=True, stderr=subprocess.PIPE, timeout=120)
    assert bad.returncode != 0


def changed(name, edit):
    c = copy.deepcopy(D.configs[name])
    edit(c)
    return c


@pytest.mark.parametrize("edit", [
    lambda c: c["layers"][0].update(type="convolution"), lambda c: c["layers"][0]["mixer"].update(kv_heads=3),
    lambda c: c["layers"][0]["mlp"].update(kind="dense"), lambda c: c["loop"].update(stop=9), lambda c: c["loop"].update(times=0),
    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=5), lambda c: c["layers"][0]["mixer"]["rot"].update(dims=32),
    lambda c: c["layers"][0]["mixer"]["rot"].update(base=0), lambda c: c["layers"][0]["mlp"]["router"].update(top=5),
    lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=3), lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(keep=5),
    lambda c: c["norm"].update(groups=5), lambda c: c["norm"].update(groups=0), lambda c: c["canon"].update(taps=0), lambda c: c.pop("token_side"),
    lambda c: c["embedding"]["bigram"].update(buckets=0), lambda c: c["embedding"].pop("bigram"), lambda c: c.pop("residual_mult"),
    lambda c: c["layers"][0]["mixer"].update(heads=2.5)], ids=range(19))
def test_configurations_that_do_not_fit(session, edit):
    with pytest.raises(RuntimeError):
        session.load_config(changed("mixed", edit))


def test_parameters_that_do_not_fit(session):
    p = C.load(D, session, "mixed")
    t = C.tokens_of(D, "mixed", 4)
    for name in ("l0.mix.talk", "l1.canon2", "l0.mlp.e3.down", "bigram", "side.embed"):
        session.set_param(name, np.eye(3, dtype=np.float32))
        with pytest.raises(RuntimeError, match=name):
            session.step(1, t)
        session.set_param(name, p[name])
    session.step(1, t)
    with pytest.raises(RuntimeError):
        session.step(1, t, rows=[4])
    session.end(1)
    session.clear_params()
    with pytest.raises(RuntimeError, match="MissingParameter"):
        session.step(1, t)
    session.end(1)
    assert session.requests_in_progress() == 0


def test_the_shapes_of_a_configuration():
    for name, c in D.configs.items():
        names = [n for n, _ in param_shapes(c)]
        assert len(names) == len(set(names))
        assert ("loop.step" in names) == bool(c["loop"]), name
        for i, l in enumerate(c["layers"]):
            assert (f"l{i}.norm2" in names) == (f"l{i}.mlp.router" in names) == bool(l["mlp"])


def test_the_pair_of_the_last_token_of_a_portion(session):
    """The first token of a portion forms a pair with the last one of the portion before; a new request's first token with none."""
    p = C.load(D, session, "no_loop")
    a, b = C.tokens_of(D, "no_loop", 9, 1), C.tokens_of(D, "no_loop", 9, 2)
    b[4:] = a[4:]
    for portions in ([4, 5], [4, 1, 4], [1] * 9):
        for t in (a, b):
            C.close(C.run(session, t, portions), D.logits("no_loop", p, t), 5e-5, f"portions {portions}")
