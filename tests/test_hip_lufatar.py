"""The Lufatar model on the GPU: prompts, portions, decoding, requests and generation against lufatar_reference.py."""
import numpy as np
import pytest

import design_cases as C
import lufatar_reference as R
from block_cases import bf16
from lufatar_cases import LUFATAR as D, decided
from catgrad_amd.lufatar import attention_layer, config_of, experts, random_params
from catgrad_amd.runner import Session

pytestmark = pytest.mark.gpu


@pytest.fixture(scope="module")
def session():
    return Session()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("how", list(C.PORTIONS))
@pytest.mark.parametrize("name", list(D.configs))
def test_portions(session, name, how, dtype):
    C.check_portions(D, session, name, how, dtype)


@pytest.mark.parametrize("name", list(D.configs))
def test_one_token(session, name):
    C.check_one_token(D, session, name)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["mixed", "wider", "odd_sizes"])
def test_interleaved_requests(session, name, dtype):
    C.check_interleaved(D, session, name, dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["mixed", "wider"])
def test_long_decode(session, name, dtype):
    C.check_long_decode(D, session, name, 260, dtype)


@pytest.mark.parametrize("name", ["mixed", "attention_only", "everything_looped", "odd_sizes", "wider"])
def test_generate(session, name):
    C.check_generate(D, session, name)


@pytest.mark.parametrize("name", ["mixed", "odd_sizes", "wider"])
def test_batch_logits(session, name):
    C.check_batch_logits(D, session, name)


def test_recorded_schedules(session):
    C.load(D, session, "mixed")
    t = C.tokens_of(D, "mixed", 30)
    want = C.run(session, t, [20, 1, 9])
    try:
        for schedule in (1, 2):
            session.set_schedule(schedule)
            np.testing.assert_allclose(C.run(session, t, [20, 1, 9]), want, rtol=1e-5, atol=1e-5)
    finally:
        session.set_schedule(0)


def test_ended_requests_give_their_memory_back(session):
    C.load(D, session, "wider")
    t = C.tokens_of(D, "wider", 120)

    def once():
        for r in range(4):
            C.run(session, t, [90] + [1] * 30, request=r, end=False)
        held = session.pool_stats()[0]
        for r in range(4):
            session.end(r)
        session.sync()
        return held, session.pool_stats()[0]

    first = once()
    assert first[0] > first[1]
    assert once()[1] == first[1]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_layers_of_a_larger_model(session, dtype):
    """Two layers at widths that take the big product tiles, a prompt cut and decoded."""
    mlp = experts(16, 4, 384, groups=4, keep=2, limit=7.0)
    c = config_of([attention_layer(16, 4, 64, 64, mlp, rot=32), attention_layer(32, 8, 64, 80, mlp, rot=64)], 1024, 1024, loop={"start": 0, "stop": 2, "times": 2},
                  side=64, buckets=997)
    p = {n: bf16(w) for n, w in (decided(random_params(c, 5), 5) if dtype == "bfloat16" else random_params(c, 5))}
    session.clear_params()
    session.load_config(c, dtype)
    for n, w in p.items():
        session.set_param(n, w)
    t = np.random.default_rng(6).integers(0, 1024, size=330)
    want = R.logits(c, p, t)
    for portions in ([330], [300] + [1] * 30, [3, 2, 130, 4, 1, 150, 12, 28]):
        C.close(C.run(session, t, portions), want, {"float32": 1e-4, "bfloat16": 4e-2}[dtype], f"portions {portions[:4]}, {dtype}")
