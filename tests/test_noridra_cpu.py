"""Noridra family on the CPU path (reference ops, fp32) against the plain
model in noridra_oracle.py: the engine's batching, paging, state slots and
scheduler with this family, and every mechanism by itself."""
import os
import sys

import pytest

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import noridra_cases as cases  # noqa: E402

DEV, DT = "cpu", "fp32"


@pytest.mark.parametrize("name", sorted(set(cases.CONFIGS) - {"tiles"}))
def test_whole_prompt(name):
    cases.case_whole(name, DEV, DT)


def test_whole_prompt_wide_heads():
    cases.case_whole("tiles", DEV, DT, n=19)


def test_residual_after_every_layer():
    cases.case_layers(DEV, DT)


@pytest.mark.parametrize("name", ["hybrid", "plain", "extreme"])
def test_prefill_against_token_by_token(name):
    cases.case_prefill_vs_decode(name, DEV, DT)


@pytest.mark.parametrize("sizes", [(2,), (3, 2, 7), (16, 1, 5)])
def test_portions(sizes):
    cases.case_portions("hybrid", DEV, DT, sizes)
    cases.case_portions("extreme", DEV, DT, sizes)


def test_unequal_batch():
    cases.case_batch("hybrid", DEV, DT)
    cases.case_batch("plain", DEV, DT)


def test_pages_and_slots_reused():
    cases.case_reuse(DEV, DT)


def test_first_tokens():
    cases.case_first_tokens(DEV, DT)


def test_long_decode():
    cases.case_long_decode(DEV, DT)


def test_long_chunk():
    cases.case_long_chunk(DEV, DT)


def test_long_portions_sort_rows_by_expert():
    cases.case_sorted_experts(DEV, DT)


@pytest.mark.parametrize("decode", [False, True])
def test_chunk_edges(decode):
    cases.case_chunk_edges(DEV, DT, decode)


@pytest.mark.parametrize("decode", [False, True])
def test_far_key(decode):
    cases.case_far_key(DEV, DT, decode)


def test_sink():
    cases.case_sink(DEV, DT)


def test_state_is_carried():
    cases.case_state_carry(DEV, DT)


def test_input_convolution():
    cases.case_input_conv(DEV, DT)


def test_router():
    cases.case_router(DEV, DT)


def test_greedy_generation():
    cases.case_generate(DEV, DT)


def test_multi_turn_and_eviction():
    cases.case_multi_turn(DEV)


def test_op_postnorm():
    cases.case_op_postnorm(DEV, DT)


def test_op_conv():
    cases.case_op_conv(DEV, DT)


def test_op_delta():
    cases.case_op_delta(DEV, DT)


def test_op_selective():
    cases.case_op_selective(DEV, DT)


def test_op_attention():
    cases.case_op_attention(DEV, DT)


def test_op_head_norm():
    cases.case_op_head_norm(DEV, DT)


def test_op_router():
    cases.case_op_router(DEV)


def test_op_experts():
    cases.case_op_experts(DEV, DT)


def test_presets_and_registry():
    from kukeon_amd.models import registry
    cfg = registry.preset("tiny-noridra")
    assert cfg.family == "noridra" and registry.family_of(cfg) == "noridra"
    model = registry.build_model(cfg, "cpu", dtype="fp32")
    assert len(model.layers) == cfg.num_layers
    assert registry.OP_GROUPS["noridra"] == ("delta",)
    big = registry.preset("noridra-8b-like")
    assert big.width == 4096 and big.num_layers == 32
    assert "noridra-8b-like" in registry.preset_names()


def test_config_rejects_what_it_does_not_know():
    for change in (lambda c: c["layers"][0].update(type="other"),
                   lambda c: c["layers"][0]["mlp"].update(kind="dense"),
                   lambda c: c["layers"][1]["mixer"].update(vdim=3)):
        cfg = cases.CONFIGS["hybrid"]()
        change(cfg)
        with pytest.raises(ValueError):
            cases.NoridraConfig.from_json(cfg)
    cfg = cases.CONFIGS["hybrid"]()
    W = cases.weights(cfg, 1)
    del W["l0.canon2"]
    with pytest.raises(KeyError):
        cases.NoridraModel(cases.NoridraConfig.from_json(cfg), device="cpu",
                           dtype="fp32", tensors=W)


def test_checkpoint_folder(tmp_path):
    cases.case_registry(tmp_path, DEV, DT)


def test_trace_runner(tmp_path):
    cases.case_trace_runner(tmp_path, DEV, DT)


def test_modelhub_server():
    cases.case_modelhub(DEV)


def test_bench_stack_shapes():
    """The throughput stack at several sizes builds its configuration (no
    weights): every layer has ff active rows."""
    from kukeon_amd.models.noridra import noridra_bench, tensor_shapes
    for W, hq, hk, ff, nl in ((2048, 16, 4, 8192, 4), (8192, 64, 8, 28672, 2)):
        cfg = noridra_bench(width=W, layers=nl, heads=hq, kv_heads=hk, ff=ff,
                            vocab=1000, max_positions=64)
        assert cfg.layers[1].type == "attention"
        for L in cfg.layers:
            assert abs(L.mlp.top * L.mlp.ff - ff) <= 16
        assert "l0.canon1" in tensor_shapes(cfg)
