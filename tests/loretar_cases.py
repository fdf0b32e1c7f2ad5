"""Small Loretar models shared by the CPU and GPU tests (what is checked on them: design_cases.py)."""
import loretar_reference as R
from design_cases import Design
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

LORETAR = Design(CONFIGS, R, lambda config, seed, name, dtype: random_params(config, seed, low_rank=5 if name == "odd_sizes" else 8), {"float32": 5e-5, "bfloat16": 4e-2})
