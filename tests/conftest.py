import os
import sys

import pytest
import torch

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
for p in (ROOT, os.path.dirname(os.path.abspath(__file__))):
    if p not in sys.path:
        sys.path.insert(0, p)


def pytest_configure(config):
    config.addinivalue_line("markers", "gpu: needs an MI355X (run with -m gpu on a GPU box)")


def pytest_collection_modifyitems(config, items):
    if torch.cuda.is_available():
        return
    skip = pytest.mark.skip(reason="no GPU in this process")
    for item in items:
        if "gpu" in item.keywords:
            item.add_marker(skip)


@pytest.fixture
def cpu_ops(monkeypatch):
    """Replaces the HIP kernels by their plain torch references, so that the engine's host logic
    (step function, cache bookkeeping, scheduler) can be exercised without a GPU.  Tests only."""
    import torch_ops
    from simply_amd.kernels import ops

    for name in ("embed", "rmsnorm", "add_rmsnorm", "rope_cache_write", "rope", "gather_rows", "fill_", "gemm",
                 "paged_attention", "sample", "score", "decode_attention_takes", "paged_attention_sink",
                 "residual_add_norm", "gated_heads", "activation_", "qk_norm_rope_cache_write", "short_conv_silu",
                 "delta_prepare", "delta_inputs", "delta_rule", "embed_sum", "token_gate_", "bias_add_", "weighted_sum",
                 "exp_gates", "linear_state", "normalized_readout", "route", "routed_experts", "residual_add_next_norm",
                 "paged_attention_maps", "attention_maps_units_takes", "norm_rope_cache_write", "short_conv", "head_product", "rglru_scan",
                 "attention_inputs", "route_choice", "token_shift", "low_rank_decay", "concat_rows", "gemm_sections"):
        monkeypatch.setattr(ops, name, getattr(torch_ops, name))
    return torch_ops


@pytest.fixture(scope="session")
def gpu_lib():
    """The built kernel library; GPU tests fail loudly if it is not there."""
    from simply_amd.kernels import lib

    lib.load()
    assert lib.library_path() is not None
    return lib
