"""The decoder blocks of the CPU oracle against the plain statements of loretar_reference.py."""
import pytest

import block_cases as C


@pytest.mark.parametrize("case", [c for c in C.LINEAR if c[0] * (c[1] + c[2]) * c[3] < 5e7], ids=str)
def test_linear(oracle, case):
    C.run_linear(oracle, case)


@pytest.mark.parametrize("case", [c for c in C.RESIDUAL if c[0] * c[1] * sum(k for k, _, _ in c[2]) < 2e7], ids=str)
def test_residual(oracle, case):
    C.run_residual(oracle, case)


@pytest.mark.parametrize("name", [n for n in C.ATTENTION if n != "keys_cut_over_workgroups"])
def test_attention(oracle, name):
    C.run_attention_case(oracle, name)


def test_attention_edges(oracle):
    C.run_attention_edges(oracle, 5, [9, 1, 1, 6])


@pytest.mark.parametrize("name", list(C.DELTA))
def test_channel_delta(oracle, name):
    C.run_delta_case(oracle, name)
