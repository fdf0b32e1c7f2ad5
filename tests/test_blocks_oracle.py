"""The decoder blocks of the CPU oracle against the plain statements of loretar_reference.py and lufatar_reference.py."""
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


@pytest.mark.parametrize("name", [n for n in C.MIXED if n not in ("keys_cut_over_workgroups", "segments_of_keys", "long_prompt_then_decode")])
def test_mixed_scores(oracle, name):
    C.run_mixed_case(oracle, name)


def test_mixed_scores_needles(oracle):
    C.run_mixed_needles(oracle, C.turned(4, 2, 16, 16, 0), [20, 1, 2, 17])


@pytest.mark.parametrize("dtype", ["f32", "bf16"])
def test_pair_embedding(oracle, dtype):
    C.run_pair_embedding(oracle, dtype)


@pytest.mark.parametrize("case", [c for c in C.CONV if sum(c[1]) * c[2] < 1e5], ids=str)
def test_conv_linear(oracle, case):
    C.run_conv_linear(oracle, case)


def test_grouped_linear(oracle):
    C.run_grouped_linear(oracle, 3, 40, 5, 7, "f32")


@pytest.mark.parametrize("case", [c for c in C.EXPERTS if c[0] * c[1] * c[3] * c[6] < 1e7], ids=str)
def test_experts(oracle, case):
    C.run_experts(oracle, case)


@pytest.mark.parametrize("rows", [1, 20])
def test_expert_choices(oracle, rows):
    C.run_expert_choices(oracle, rows)


@pytest.mark.parametrize("case", [c for c in C.SIDE if c[0] * c[1] < 1e5], ids=str)
def test_token_side(oracle, case):
    C.run_side(oracle, case)
