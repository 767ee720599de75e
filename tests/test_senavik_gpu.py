"""Senavik family on an MI355X: the HIP kernels, in exact fp32 mode and in
the bf16 serving mode, against the plain model in senavik_oracle.py."""
import os
import sys

import pytest

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import senavik_cases as cases  # noqa: E402

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
BOTH = pytest.mark.parametrize("dtype", ["fp32", "bf16"])
KINDS = pytest.mark.parametrize("kind", ["attention", "latent_attention"])


def test_kernel_group_is_loaded():
    from kukeon_amd import ops
    assert ops.sink_available(), "kukeon_amd/_C_sink.so is not built"


@BOTH
def test_op_norms(dtype):
    cases.case_op_norms(DEV, dtype)


@BOTH
def test_op_rotary(dtype):
    cases.case_op_rotary(DEV, dtype)


@BOTH
@pytest.mark.parametrize("d,dv,BS", [(8, 8, 4), (7, 11, 4), (96, 40, 16),
                                     (24, 128, 16), (128, 128, 16)])
def test_op_attention(d, dv, BS, dtype):
    cases.case_op_attention(DEV, dtype, d, dv, BS)
    cases.case_op_attention(DEV, dtype, d, dv, BS, n=101, start=60)


@BOTH
@pytest.mark.parametrize("sizes", [
    (5, 24, 6), (3, 300, 8), (2, 520, 4), (6, 64, 16), (4, 128, 8),
    (20, 128, 32), (3, 256, 64), (17, 512, 64)])
def test_op_latent(sizes, dtype):
    cases.case_op_latent(DEV, dtype, *sizes)
    # enough keys that few rows share them out over several workgroups
    cases.case_op_latent(DEV, dtype, *sizes, n=700, BS=16,
                         rows=[0, 255, 256, 300, 512, 699])


@BOTH
def test_op_heads(dtype):
    cases.case_op_heads(DEV, dtype)


def test_op_router():
    cases.case_op_router(DEV)


@BOTH
@pytest.mark.parametrize("name", sorted(cases.CONFIGS))
def test_whole_prompt(name, dtype):
    cases.case_whole(name, DEV, dtype)


@BOTH
def test_residual_after_every_layer(dtype):
    cases.case_layers(DEV, dtype)


@BOTH
@pytest.mark.parametrize("name", ["hybrid", "aligned", "plain", "extreme"])
def test_prefill_against_token_by_token(name, dtype):
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
def test_pages_reused(dtype):
    cases.case_reuse(DEV, dtype)


@BOTH
def test_first_tokens(dtype):
    cases.case_first_tokens(DEV, dtype)


@BOTH
def test_long_decode(dtype):
    cases.case_long_decode(DEV, dtype)


@BOTH
def test_long_window(dtype):
    cases.case_long_window(DEV, dtype)


@BOTH
def test_long_portions(dtype):
    cases.case_long_portions(DEV, dtype)


@BOTH
def test_long_portions_sort_rows_by_expert(dtype):
    cases.case_sorted_experts(DEV, dtype)


@BOTH
@pytest.mark.parametrize("decode", [False, True])
def test_window_edges(decode, dtype):
    cases.case_window_edges(DEV, dtype, decode)
    # heads and pages of the matrix-core kernel
    cases.case_window_edges(DEV, dtype, decode, dim=128, vdim=128, bs=16)


@BOTH
@KINDS
@pytest.mark.parametrize("decode", [False, True])
def test_far_key(kind, decode, dtype):
    cases.case_far_key(kind, DEV, dtype, decode)
    cases.case_far_key(kind, DEV, dtype, decode, dim=128)


@BOTH
@KINDS
def test_sink(kind, dtype):
    cases.case_sink(kind, DEV, dtype)
    cases.case_sink(kind, DEV, dtype, dim=128)


@BOTH
def test_feed_forwards(dtype):
    cases.case_feed_forwards(DEV, dtype)


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
