"""Token language models on a real MI355X: the cases of tests/tlm_cases.py through libmoshi_tlm.so (hipGraph replay in decode steps)."""
import pytest

from tests import tlm_cases as tc

pytestmark = pytest.mark.gpu
DEV = "cuda"


@pytest.fixture(scope="session")
def lib():
    import torch
    assert torch.cuda.is_available(), "-m gpu tests need a GPU"
    from moshi_amd import _capi
    return _capi.load_tlm()


@pytest.mark.parametrize("dtype", [tc.F32, tc.BF16], ids=["fp32", "bf16"])
@pytest.mark.parametrize("name", sorted(tc.MECHANISMS))
def test_mechanism(lib, name, dtype):
    tc.check_mechanism(name, DEV, lib, dtype)


def test_activation_branches(lib):
    tc.check_activation_branches(DEV, lib)


@pytest.mark.parametrize("dtype", [tc.F32, tc.BF16], ids=["fp32", "bf16"])
@pytest.mark.parametrize("case", ["portions", "prompt_then_decode", "unequal_batch", "batched_decode", "reuse", "long_decode", "long_prompt", "first_tokens"])
def test_feeding(lib, case, dtype):
    getattr(tc, f"check_{case}")(DEV, lib, dtype)


@pytest.mark.parametrize("dtype", [tc.F32, tc.BF16], ids=["fp32", "bf16"])
@pytest.mark.parametrize("name", sorted(tc.WIDE_PROMPTS))
def test_long_prompt_per_latent_width(lib, name, dtype):
    tc.check_long_prompt(DEV, lib, dtype, n=700, cfg=tc.WIDE_PROMPTS[name])


@pytest.mark.parametrize("dtype", [tc.F32, tc.BF16], ids=["fp32", "bf16"])
@pytest.mark.parametrize("case", ["portions", "prompt_then_decode", "unequal_batch", "batched_decode", "reuse", "first_tokens"])
def test_feeding_bibapel(lib, case, dtype):
    getattr(tc, f"check_{case}")(DEV, lib, dtype, name="bibapel")


@pytest.mark.parametrize("dtype", [tc.F32, tc.BF16], ids=["fp32", "bf16"])
def test_decoding_longer_than_the_pool_with_kept_pages(lib, dtype):
    tc.check_long_decode(DEV, lib, dtype, name="two_kept_windows", n=700, held=4)


@pytest.mark.parametrize("dtype", [tc.F32, tc.BF16], ids=["fp32", "bf16"])
@pytest.mark.parametrize("name", sorted(tc.WIDE_PROMPTS_2))
def test_long_prompt_per_head_size(lib, name, dtype):
    tc.check_long_prompt(DEV, lib, dtype, n=800, cfg=tc.WIDE_PROMPTS_2[name])


@pytest.mark.parametrize("dtype", [tc.F32, tc.BF16], ids=["fp32", "bf16"])
@pytest.mark.parametrize("name", sorted(tc.BESIDE))
def test_long_prompt_beside_decoding(lib, name, dtype):
    tc.check_long_prompt_beside_decoding(DEV, lib, dtype, n=900, name=name)


@pytest.mark.parametrize("window,keep", [(70, 7), (64, 1), (33, 64), (0, 0)])
def test_single_kept_keys(lib, window, keep):
    tc.check_single_kept_keys(DEV, lib, window, keep)


@pytest.mark.parametrize("case", ["sink", "matrix_state_far", "decay_extremes", "glu_limits", "previous_token", "last_position"])
def test_single_mechanisms(lib, case):
    getattr(tc, f"check_{case}")(DEV, lib)


def test_greedy_generation_through_the_scheduler_bibapel(lib):
    tc.check_generation(DEV, lib, name="bibapel")


@pytest.mark.parametrize("window", [70, 64, 0])
def test_single_keys(lib, window):
    tc.check_single_keys(DEV, lib, window)


def test_state_reaches_far_back(lib):
    tc.check_far_state(DEV, lib)


def test_greedy_generation_through_the_scheduler(lib):
    tc.check_generation(DEV, lib)


def test_sampling(lib):
    tc.check_sampling(DEV, lib)


def test_limits_and_errors(lib):
    tc.check_limits(DEV, lib)


def test_trace_replay(lib, tmp_path):
    tc.check_replay(DEV, lib, tmp_path)
