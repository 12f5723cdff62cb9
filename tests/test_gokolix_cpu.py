"""Gokolix on the CPU: the engine's host logic (ragged scheduling, pages, state slots, checkpoint placement) with the
package's torch restatement of the kernels, against the oracle."""
import pytest

from tests import _gokolix as K
from tests import _gokolix_cases as C

DEV = "cpu"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_mechanisms(dtype):
    C.case_embedding_and_split(DEV, dtype)
    C.case_head_norm_store(DEV, dtype)
    C.case_latent_store(DEV, dtype)
    C.case_recurrence(DEV, dtype)
    C.case_windowed_latent_attention(DEV, dtype)
    C.case_gated_relu(DEV, dtype)


def test_yarn_and_bias_tables():
    C.case_yarn_and_bias_tables(DEV)


def test_extended_attention():
    C.case_extended_attention(DEV, "float32")


def test_recurrence_long_and_many():
    C.case_recurrence_long_and_many(DEV, "float32")


def test_checkpoint_placement(tmp_path):
    C.case_checkpoint_placement(tmp_path)


@pytest.mark.parametrize("name", ["CFG_MAIN", "CFG_ODD", "CFG_WIDE"])
def test_layer_by_layer(tmp_path, name):
    C.case_layer_by_layer(DEV, tmp_path, cfg=getattr(K, name))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_engine_schedules(tmp_path, dtype):
    C.case_engine_schedules(DEV, dtype, tmp_path)


@pytest.mark.parametrize("name", ["CFG_ODD", "CFG_WIDE", "CFG_ONE", "CFG_ONE_LRU"])
def test_engine_other_sizes(tmp_path, name):
    C.case_engine_schedules(DEV, "float32", tmp_path, cfg=getattr(K, name), seed=9)


@pytest.mark.parametrize("seed", [301, 304])
def test_engine_random_configs(tmp_path, seed):
    C.case_engine_random_config(DEV, "float32", tmp_path, seed)


def test_engine_long(tmp_path):
    C.case_engine_long(DEV, "float32", tmp_path)


def test_engine_far_token(tmp_path):
    C.case_engine_far_token(DEV, tmp_path)


def test_engine_reuse_of_pages_and_slots(tmp_path):
    C.case_engine_reuse(DEV, "float32", tmp_path)


def test_engine_long_decode(tmp_path):
    C.case_engine_long_decode(DEV, "float32", tmp_path)


def test_generate(tmp_path):
    C.case_generate(DEV, tmp_path)


def test_generate_under_preemption(tmp_path):
    C.case_generate_preemption(DEV, tmp_path)
