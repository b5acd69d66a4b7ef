"""Token language models on the kernel simulator: the cases of tests/tlm_cases.py, and bit-identical results under perturbed schedules."""
import os
import sys

import numpy as np
import pytest

from tests import tlm_cases as tc
from tests.conftest import ROOT

DEV = "cpu"


@pytest.fixture(scope="session")
def tlm_lib():
    os.environ["MMI_NO_GRAPH"] = "1"
    sys.path.insert(0, str(ROOT / "tests" / "hipsim"))
    import build_sim
    from moshi_amd import _capi
    return _capi.load_tlm(os.environ.get("MMI_TLM_SIM_LIB") or build_sim.build_tlm())


@pytest.mark.parametrize("name", sorted(tc.MECHANISMS))
def test_mechanism_fp32(tlm_lib, name):
    tc.check_mechanism(name, DEV, tlm_lib)


@pytest.mark.parametrize("name", ["mingru_experts", "attention_experts", "wide_latent", "repeated", "mixed", "grouped_attention", "delta", "lightning", "glu",
                                  "projected_passes", "bibapel"])
def test_mechanism_bf16(tlm_lib, name):
    tc.check_mechanism(name, DEV, tlm_lib, tc.BF16)


def test_activation_branches(tlm_lib):
    tc.check_activation_branches(DEV, tlm_lib)


def test_portions_of_a_prompt(tlm_lib):
    tc.check_portions(DEV, tlm_lib)


def test_portions_of_a_prompt_bf16(tlm_lib):
    tc.check_portions(DEV, tlm_lib, tc.BF16, n=100, cut_sets=((2,), (65, 1)))


def test_prompt_then_decode(tlm_lib):
    tc.check_prompt_then_decode(DEV, tlm_lib)


def test_unequal_requests_in_one_batch(tlm_lib):
    tc.check_unequal_batch(DEV, tlm_lib)


def test_batched_decode(tlm_lib):
    tc.check_batched_decode(DEV, tlm_lib, steps=4)


def test_pages_and_slots_are_used_again(tlm_lib):
    tc.check_reuse(DEV, tlm_lib)


def test_decoding_longer_than_the_pool(tlm_lib):
    tc.check_long_decode(DEV, tlm_lib)


def test_long_prompt(tlm_lib):
    tc.check_long_prompt(DEV, tlm_lib)


@pytest.mark.parametrize("window", [70, 64, 0])
def test_single_keys(tlm_lib, window):
    tc.check_single_keys(DEV, tlm_lib, window)


def test_state_reaches_far_back(tlm_lib):
    tc.check_far_state(DEV, tlm_lib)


def test_first_tokens(tlm_lib):
    tc.check_first_tokens(DEV, tlm_lib)


def test_greedy_generation_through_the_scheduler(tlm_lib):
    tc.check_generation(DEV, tlm_lib)


def test_sampling(tlm_lib):
    tc.check_sampling(DEV, tlm_lib)


def test_limits_and_errors(tlm_lib):
    tc.check_limits(DEV, tlm_lib)


def test_trace_replay(tlm_lib, tmp_path):
    tc.check_replay(DEV, tlm_lib, tmp_path)


# ---- the mixers with matrix states, grouped attention, and the network that has them all -------------------------------------------
def test_portions_of_a_prompt_bibapel(tlm_lib):
    tc.check_portions(DEV, tlm_lib, n=100, cut_sets=((2,), (3, 2, 61, 7), (65, 1), (5,)), name="bibapel")


def test_prompt_then_decode_bibapel(tlm_lib):
    tc.check_prompt_then_decode(DEV, tlm_lib, n=90, tail=20, name="bibapel")


def test_unequal_requests_in_one_batch_bibapel(tlm_lib):
    tc.check_unequal_batch(DEV, tlm_lib, name="bibapel")


def test_long_prompt_beside_decoding(tlm_lib):
    tc.check_long_prompt_beside_decoding(DEV, tlm_lib, name="all")


def test_batched_decode_bibapel(tlm_lib):
    tc.check_batched_decode(DEV, tlm_lib, steps=4, name="bibapel")


def test_pages_and_slots_are_used_again_bibapel(tlm_lib):
    tc.check_reuse(DEV, tlm_lib, name="bibapel")


def test_decoding_longer_than_the_pool_with_kept_pages(tlm_lib):
    tc.check_long_decode(DEV, tlm_lib, name="two_kept_windows", n=400, held=4)


@pytest.mark.parametrize("window,keep", [(70, 7), (64, 1), (33, 64), (0, 0)])
def test_single_kept_keys(tlm_lib, window, keep):
    tc.check_single_kept_keys(DEV, tlm_lib, window, keep, queries=(128, 103) if window else (128,))


@pytest.mark.parametrize("case", ["sink", "matrix_state_far", "decay_extremes", "glu_limits", "previous_token", "last_position"])
def test_single_mechanisms(tlm_lib, case):
    getattr(tc, f"check_{case}")(DEV, tlm_lib)


def test_first_tokens_bibapel(tlm_lib):
    tc.check_first_tokens(DEV, tlm_lib, name="bibapel")


def test_greedy_generation_through_the_scheduler_bibapel(tlm_lib):
    tc.check_generation(DEV, tlm_lib, name="bibapel")


@pytest.mark.parametrize("name", ["mixed", "bibapel"])
def test_perturbed_schedules_give_the_same_bits(tlm_lib, name):
    """Waves and lanes of a workgroup in other orders (a missing barrier would show); the order of a routed expert's pairs comes from
    atomics and must not matter either."""
    cfg = tc.MECHANISMS[name]
    toks = tc.tokens_of(cfg, 80)

    def run(mode, seed):
        tlm_lib.cdll.hipsim_set_schedule(mode, seed)
        try:
            return [tc.run_cut(tc.make(cfg, DEV, tlm_lib, dt)[0], toks, [70, 1, 9]) for dt in (tc.F32, tc.BF16)]
        finally:
            tlm_lib.cdll.hipsim_set_schedule(0, 1)
    want = run(0, 1)
    for mode, seed in ((1, 1), (2, 7)):
        for a, b in zip(run(mode, seed), want):
            assert np.array_equal(a, b), (mode, seed)
