"""Gokolix on the GPU: the HIP kernels of liblvmix.so, alone and through the engine, against the oracle."""
import pytest

from tests import _gokolix as K
from tests import _gokolix_cases as C

pytestmark = pytest.mark.gpu
DEV = "cuda"
DTYPES = ["float32", "bfloat16"]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", [C.case_embedding_and_split, C.case_head_norm_store, C.case_latent_store, C.case_extended_attention,
                                  C.case_windowed_latent_attention, C.case_recurrence, C.case_recurrence_long_and_many, C.case_gated_relu],
                         ids=lambda c: c.__name__[5:])
def test_mechanism(gpu, case, dtype):
    case(DEV, dtype)


def test_yarn_and_bias_tables(gpu):
    C.case_yarn_and_bias_tables(DEV)


def test_vector_attention_agrees_with_the_matrix_cores(gpu):
    """The same bf16 cases with the vector kernel forced: both kernels read the same factors, biases and sinks."""
    from light_vllm_amd import mix_ops
    old, mix_ops.WINDOW_ATTN_KERNEL = mix_ops.WINDOW_ATTN_KERNEL, "valu"
    try:
        C.case_extended_attention(DEV, "bfloat16")
    finally:
        mix_ops.WINDOW_ATTN_KERNEL = old


@pytest.mark.parametrize("name", ["CFG_MAIN", "CFG_ODD", "CFG_WIDE"])
def test_layer_by_layer(gpu, tmp_path, name):
    C.case_layer_by_layer(DEV, tmp_path, cfg=getattr(K, name))


@pytest.mark.parametrize("dtype", DTYPES)
def test_engine_schedules(gpu, tmp_path, dtype):
    C.case_engine_schedules(DEV, dtype, tmp_path)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["CFG_ODD", "CFG_WIDE", "CFG_ONE", "CFG_ONE_LRU"])
def test_engine_other_sizes(gpu, tmp_path, name, dtype):
    C.case_engine_schedules(DEV, dtype, tmp_path, cfg=getattr(K, name), seed=9)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("seed", [301, 302, 303, 304, 305, 306])
def test_engine_random_configs(gpu, tmp_path, seed, dtype):
    C.case_engine_random_config(DEV, dtype, tmp_path, seed)


@pytest.mark.parametrize("dtype", DTYPES)
def test_engine_long(gpu, tmp_path, dtype):
    C.case_engine_long(DEV, dtype, tmp_path)


def test_engine_far_token(gpu, tmp_path):
    C.case_engine_far_token(DEV, tmp_path)


@pytest.mark.parametrize("dtype", DTYPES)
def test_engine_reuse_of_pages_and_slots(gpu, tmp_path, dtype):
    C.case_engine_reuse(DEV, dtype, tmp_path)


@pytest.mark.parametrize("dtype", DTYPES)
def test_engine_long_decode(gpu, tmp_path, dtype):
    C.case_engine_long_decode(DEV, dtype, tmp_path)


def test_generate(gpu, tmp_path):
    C.case_generate(DEV, tmp_path)


def test_generate_from_graphs(gpu, tmp_path):
    C.case_generate(DEV, tmp_path, enforce_eager=False)


def test_generate_bf16_graphs_like_eager(gpu, tmp_path):
    C.case_generate_bf16_graphs_like_eager(DEV, tmp_path)


def test_generate_under_preemption(gpu, tmp_path):
    C.case_generate_preemption(DEV, tmp_path)
