"""Noridra family on an MI355X: the HIP kernels, in exact fp32 mode and in
the bf16 serving mode, against the plain model in noridra_oracle.py."""
import os
import sys

import pytest

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import noridra_cases as cases  # noqa: E402

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
BOTH = pytest.mark.parametrize("dtype", ["fp32", "bf16"])


def test_kernel_group_is_loaded():
    from kukeon_amd import ops
    assert ops.delta_available(), "kukeon_amd/_C_delta.so is not built"


@BOTH
def test_op_postnorm(dtype):
    cases.case_op_postnorm(DEV, dtype)


@BOTH
def test_op_conv(dtype):
    cases.case_op_conv(DEV, dtype)


@BOTH
@pytest.mark.parametrize("sizes", [
    (4, 2, 5, 7), (2, 2, 32, 64), (3, 1, 64, 24), (2, 1, 128, 128),
    (1, 1, 160, 20), (2, 2, 260, 18), (6, 2, 40, 33)])
def test_op_delta(sizes, dtype):
    cases.case_op_delta(DEV, dtype, *sizes)
    # more than one tile of tokens
    cases.case_op_delta(DEV, dtype, *sizes, cuts=(37, 1, 3, 16, 2))


@BOTH
@pytest.mark.parametrize("sizes", [(9, 5), (24, 1), (300, 8), (64, 16),
                                   (40, 24), (17, 40), (33, 70), (20, 128),
                                   (12, 200)])
def test_op_selective(sizes, dtype):
    cases.case_op_selective(DEV, dtype, *sizes)
    cases.case_op_selective(DEV, dtype, *sizes, cuts=(70, 1, 3, 33, 2))


@pytest.mark.parametrize("N", [8, 16, 24, 64, 100])
def test_op_selective_many_channels(N):
    """Enough channels that each keeps its states in few threads."""
    cases.case_op_selective(DEV, "fp32", 70000, N, cuts=(5, 2))


@BOTH
@pytest.mark.parametrize("d,BS", [(8, 4), (7, 4), (96, 16), (128, 16)])
def test_op_attention(d, BS, dtype):
    cases.case_op_attention(DEV, dtype, d, BS)
    cases.case_op_attention(DEV, dtype, d, BS, n=101, start=60)


@BOTH
def test_op_head_norm(dtype):
    cases.case_op_head_norm(DEV, dtype)


def test_op_router():
    cases.case_op_router(DEV)


@BOTH
def test_op_experts(dtype):
    cases.case_op_experts(DEV, dtype)


@BOTH
@pytest.mark.parametrize("name", sorted(cases.CONFIGS))
def test_whole_prompt(name, dtype):
    if name == "extreme" and dtype == "bf16":
        pytest.skip("runs of one entry turn rounding into signs")
    cases.case_whole(name, DEV, dtype)


@BOTH
def test_residual_after_every_layer(dtype):
    cases.case_layers(DEV, dtype)


@BOTH
@pytest.mark.parametrize("name", ["hybrid", "aligned", "plain", "extreme",
                                  "wide"])
def test_prefill_against_token_by_token(name, dtype):
    if name == "extreme" and dtype == "bf16":
        pytest.skip("runs of one entry turn rounding into signs")
    cases.case_prefill_vs_decode(name, DEV, dtype)


@BOTH
@pytest.mark.parametrize("sizes", [(2,), (3, 2, 7), (16, 1, 5)])
def test_portions(sizes, dtype):
    cases.case_portions("hybrid", DEV, dtype, sizes)
    cases.case_portions("aligned", DEV, dtype, sizes)


@BOTH
@pytest.mark.parametrize("name", ["hybrid", "aligned", "plain"])
def test_unequal_batch(name, dtype):
    cases.case_batch(name, DEV, dtype)


@BOTH
def test_pages_and_slots_reused(dtype):
    cases.case_reuse(DEV, dtype)


@BOTH
def test_first_tokens(dtype):
    cases.case_first_tokens(DEV, dtype)


@BOTH
def test_long_decode(dtype):
    cases.case_long_decode(DEV, dtype)


@BOTH
def test_long_chunk(dtype):
    cases.case_long_chunk(DEV, dtype)


@BOTH
def test_long_portions(dtype):
    cases.case_long_portions(DEV, dtype)


@BOTH
def test_long_portions_sort_rows_by_expert(dtype):
    cases.case_sorted_experts(DEV, dtype)


@BOTH
@pytest.mark.parametrize("decode", [False, True])
def test_chunk_edges(decode, dtype):
    cases.case_chunk_edges(DEV, dtype, decode)
    # heads and pages of the matrix-core kernel
    cases.case_chunk_edges(DEV, dtype, decode, dim=128, bs=16)


@BOTH
@pytest.mark.parametrize("decode", [False, True])
def test_far_key(decode, dtype):
    cases.case_far_key(DEV, dtype, decode)


@BOTH
def test_sink(dtype):
    cases.case_sink(DEV, dtype)


@BOTH
def test_state_is_carried(dtype):
    cases.case_state_carry(DEV, dtype)


@BOTH
def test_input_convolution(dtype):
    cases.case_input_conv(DEV, dtype)


@BOTH
def test_router(dtype):
    cases.case_router(DEV, dtype)


@BOTH
@pytest.mark.parametrize("graphs", [False, True])
def test_greedy_generation(graphs, dtype):
    cases.case_generate(DEV, dtype, use_graphs=graphs)


@BOTH
def test_graph_replays(dtype):
    cases.case_graph_replays(DEV, dtype)


def test_multi_turn_and_eviction():
    cases.case_multi_turn(DEV)


def test_checkpoint_folder(tmp_path):
    cases.case_registry(tmp_path, DEV, "bf16")


@BOTH
def test_trace_runner(tmp_path, dtype):
    cases.case_trace_runner(tmp_path, DEV, dtype)


def test_modelhub_server():
    cases.case_modelhub(DEV)


def test_real_sizes():
    def say(s):
        print("real sizes:", s, flush=True)
    cases.case_real_sizes(DEV, say)
