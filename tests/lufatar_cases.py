"""Small Lufatar models shared by the CPU and GPU tests (what is checked on them: design_cases.py)."""
import numpy as np

import lufatar_reference as R
from catgrad_amd.lufatar import attention_layer, config_of, experts, random_params
from design_cases import Design


def layers_mixed():
    return [attention_layer(4, 2, 16, 20, experts(8, 2, 24, groups=4, keep=2), rot=8), attention_layer(6, 3, 8, 12, experts(6, 3, 16, limit=0.8), rot=8, base=500.0),
            attention_layer(4, 4, 12, 8, None, rot=4, scale=0.6), attention_layer(2, 1, 24, 16, experts(9, 2, 32, groups=3, keep=1), rot=24)]


CONFIGS = {
    "mixed": config_of(layers_mixed(), 71, 64, loop={"start": 1, "stop": 3, "times": 2}, eps=1e-4, mult=0.7, side=12),
    "no_loop": config_of(layers_mixed(), 64, 32, groups=2, eps=1e-5),
    "everything_looped": config_of(layers_mixed()[:3], 50, 48, loop={"start": 0, "stop": 3, "times": 3}, mult=1.0, taps=3, side=24),
    "a_loop_of_one_pass": config_of(layers_mixed()[:2], 50, 48, loop={"start": 1, "stop": 2, "times": 1}, groups=6),
    "looped_to_the_end": config_of(layers_mixed(), 50, 40, loop={"start": 2, "stop": 4, "times": 2}, taps=2, side=8),
    "odd_sizes": config_of([attention_layer(3, 1, 10, 7, experts(5, 2, 13), rot=6), attention_layer(3, 3, 14, 5, experts(6, 4, 9, groups=2, keep=2), rot=2)], 37, 30,
                           loop={"start": 0, "stop": 1, "times": 2}, groups=3, side=7, taps=5, buckets=7, mul_prev=1009, mul_cur=70001),
    "one_of_each": config_of([attention_layer(1, 1, 8, 8, experts(1, 1, 8), rot=2)], 23, 16, groups=1, taps=1, side=4, buckets=1, mul_prev=1, mul_cur=1),
    "attention_only": config_of([attention_layer(8, 2, 16, 16, None, rot=16), attention_layer(2, 1, 32, 8, None, rot=0)], 64, 32),
    "single_members": config_of([attention_layer(4, 2, 16, 16, experts(4, 2, 24, groups=4, keep=3), rot=8)] * 2, 41, 32, groups=8),
    "all_experts": config_of([attention_layer(4, 2, 16, 16, experts(4, 4, 24, groups=2, keep=2), rot=8)], 41, 32, taps=8),
    "wider": config_of([attention_layer(10, 5, 32, 40, experts(12, 3, 88, groups=4, keep=2, limit=7.0), rot=16, base=1e5)] * 2, 300, 160,
                       loop={"start": 0, "stop": 2, "times": 2}, side=32, buckets=251, mul_prev=101, mul_cur=13),
}


def decided(params, seed):
    """Corrections so far apart that no rounding changes a choice: products of bfloat16 weights can be compared then."""
    rng = np.random.default_rng(seed)
    for n, w in params:
        yield n, (2.5 * 2.0 ** rng.permutation(len(w)) - 60.0).astype(np.float32) if n.endswith(".correction") else w


def params(config, seed, name, dtype):
    p = random_params(config, seed)
    return decided(p, seed) if dtype == "bfloat16" else p


LUFATAR = Design(CONFIGS, R, params, {"float32": 5e-5, "bfloat16": 4e-2})
