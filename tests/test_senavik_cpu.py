"""Senavik family on the CPU path (reference ops, fp32) against the plain
model in senavik_oracle.py: the engine's batching, paging and scheduler with
this family, and every mechanism by itself."""
import os
import sys

import pytest

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import senavik_cases as cases  # noqa: E402

DEV, DT = "cpu", "fp32"
KINDS = pytest.mark.parametrize("kind", ["attention", "latent_attention"])


@pytest.mark.parametrize("name", sorted(cases.CONFIGS))
def test_whole_prompt(name):
    cases.case_whole(name, DEV, DT)


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


def test_pages_reused():
    cases.case_reuse(DEV, DT)


def test_first_tokens():
    cases.case_first_tokens(DEV, DT)


def test_long_decode():
    cases.case_long_decode(DEV, DT)


def test_long_window():
    cases.case_long_window(DEV, DT)


def test_long_portions_sort_rows_by_expert():
    cases.case_sorted_experts(DEV, DT)


@pytest.mark.parametrize("decode", [False, True])
def test_window_edges(decode):
    cases.case_window_edges(DEV, DT, decode)


@KINDS
def test_far_key(kind):
    cases.case_far_key(kind, DEV, DT, True)


@KINDS
def test_sink(kind):
    cases.case_sink(kind, DEV, DT)


def test_random_weights_hide_no_fault():
    cases.case_faults_show()


def test_rotation_tables():
    cases.case_rotation_tables()


def test_feed_forwards():
    cases.case_feed_forwards(DEV, DT)


def test_greedy_generation():
    cases.case_generate(DEV, DT)


def test_multi_turn_and_eviction():
    cases.case_multi_turn(DEV)


def test_op_norms():
    cases.case_op_norms(DEV, DT)


def test_op_rotary():
    cases.case_op_rotary(DEV, DT)


def test_op_attention():
    cases.case_op_attention(DEV, DT)
    cases.case_op_attention(DEV, DT, 6, 11, n=80, start=61)


def test_op_latent():
    cases.case_op_latent(DEV, DT)


def test_op_heads():
    cases.case_op_heads(DEV, DT)


def test_op_router():
    cases.case_op_router(DEV)


def test_presets_and_registry():
    from kukeon_amd.models import registry
    cfg = registry.preset("tiny-senavik")
    assert cfg.family == "senavik" and registry.family_of(cfg) == "senavik"
    model = registry.build_model(cfg, "cpu", dtype="fp32")
    assert len(model.layers) == cfg.num_layers
    assert registry.OP_GROUPS["senavik"] == ("sink",)
    big = registry.preset("senavik-8b-like")
    assert big.width == 4096 and big.num_layers == 32
    assert "senavik-8b-like" in registry.preset_names()
    with pytest.raises(KeyError):
        registry.preset("no-such-model")


def test_config_rejects_what_it_does_not_know():
    for change in (lambda c: c["layers"][0].update(type="other"),
                   lambda c: c["layers"][1]["mlp"].update(kind="other")):
        cfg = cases.CONFIGS["hybrid"]()
        change(cfg)
        with pytest.raises(ValueError):
            cases.SenavikConfig.from_json(cfg)
    for change in (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=12),
                   lambda c: c["layers"][0]["mixer"].update(kv_heads=3),
                   lambda c: c["layers"][0]["mlp"]["router"].update(
                       groups={"count": 4, "keep": 1})):
        cfg = cases.CONFIGS["hybrid"]()
        W = cases.weights(cfg, 1)
        change(cfg)
        with pytest.raises((ValueError, KeyError)):
            cases.SenavikModel(cases.SenavikConfig.from_json(cfg),
                               device="cpu", dtype="fp32", tensors=W)
    cfg = cases.CONFIGS["hybrid"]()
    W = cases.weights(cfg, 1)
    del W["l0.mix.sink"]
    with pytest.raises(KeyError):
        cases.SenavikModel(cases.SenavikConfig.from_json(cfg), device="cpu",
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
    from kukeon_amd.models.senavik import senavik_bench, tensor_shapes
    for W, hq, hk, ff, nl in ((2048, 16, 4, 8192, 4), (8192, 64, 8, 28672, 4)):
        cfg = senavik_bench(width=W, layers=nl, heads=hq, kv_heads=hk, ff=ff,
                            vocab=1000)
        assert cfg.layers[3].type == "latent_attention"
        for L in cfg.layers:
            assert abs(max(L.mlp.top, 1) * L.mlp.ff - ff) <= 16
        assert "l1.mlp.correction" in tensor_shapes(cfg)
