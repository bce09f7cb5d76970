"""Nozizen on the GPU: every kernel against the plain implementation's function for its mechanism, the mixers and
feed-forwards as parts, and the engine (whole prompts, token-by-token decoding, portions down to two tokens, unequal
requests together in a tight pool, long decoding, recorded decode steps, greedy generation through the scheduler, trace
replay as a child process) against the plain implementation, in 32-bit and in bfloat16."""
import pytest
import torch

import nozizen_cases as cases
import nozizen_mechanisms as mech
import plain_nozizen as plain
from simply_amd.engine import StepEntry
from simply_amd.kernels import ops

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = [torch.float32, torch.bfloat16]


@pytest.fixture(autouse=True)
def _lib(gpu_lib):
    return gpu_lib


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("body", [mech.streams, mech.convolution_and_gates, mech.group_norm_behind_a_gate, mech.rotated_inputs])
def test_kernel(body, dtype):
    body(ops, DEV, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("pieces", [False, True])
def test_recurrence(dtype, pieces):
    mech.recurrence_of_groups(ops, DEV, dtype, pieces)
    mech.far_token_in_the_recurrence(ops, DEV, dtype, pieces)


def test_router():
    mech.router_among_the_chosen(ops, DEV)


def test_streams_from_partial_sums():
    mech.streams_from_partial_sums(ops, DEV)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("body", [mech.streams_block, mech.state_space_part, mech.wkv_part, mech.attention_part, mech.routed_part,
                                  mech.dense_part])
def test_part(body, dtype):
    body(DEV, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_parts_at_other_sizes(dtype):
    mech.state_space_part(DEV, dtype, sizes=(24, 1, 1, 1, 1, 1, 1), length=9, cuts=([9], [2, 2, 2, 2, 1], [1] * 9))
    mech.state_space_part(DEV, dtype, sizes=(24, 6, 3, 4, 8, 8, 2), length=40, cuts=([40], [2, 13, 2, 23], [1] * 40))
    mech.state_space_part(DEV, dtype, sizes=(24, 2, 1, 8, 200, 4, 1), length=40, cuts=([40], [2, 13, 2, 23], [1] * 40))
    mech.attention_part(DEV, dtype, sizes=(24, 3, 3, 4, 4), window=1, rot=None, length=12, cuts=([12], [5, 2, 5], [1] * 12))
    mech.attention_part(DEV, dtype, sizes=(24, 4, 1, 8, 2), window=None, rot=mech.ROTATIONS[3], length=30, cuts=([30], [1] * 30))
    mech.routed_part(DEV, dtype, experts=4, top=4, T=9)
    mech.routed_part(DEV, dtype, experts=4, top=2, ff=64, width=64, T=200)


def test_parts_at_aligned_sizes():
    """Sizes in multiples of 16, 32 and 64 in pages of 16 keys, bfloat16, 300 tokens: whatever fast kernels the parts choose
    at such sizes, whole, decoding behind a long portion, and in portions of 17."""
    cuts = ([300], [268] + [1] * 32, [17] * 17 + [11])
    mech.state_space_part(DEV, torch.bfloat16, sizes=(128, 4, 2, 32, 64, 4, 2), length=300, cuts=cuts, std=0.1)
    mech.state_space_part(DEV, torch.bfloat16, sizes=(256, 8, 1, 64, 128, 4, 8), length=300, cuts=cuts, std=0.08)
    for sizes, window, rot in (((128, 8, 2, 64, 64), 100, mech.ROTATIONS[2]), ((128, 8, 4, 96, 64), 37, mech.ROTATIONS[2]),
                               ((128, 6, 2, 32, 48), None, mech.ROTATIONS[0]), ((128, 16, 1, 128, 128), 64, mech.ROTATIONS[2]),
                               ((128, 3, 1, 160, 112), 129, mech.ROTATIONS[2])):
        mech.attention_part(DEV, torch.bfloat16, sizes=sizes, window=window, rot=rot, page_size=16, length=300, cuts=cuts, std=0.1)


def test_heads_filled_up_for_the_matrix_cores():
    """Head sizes that the bfloat16 matrix-core kernels do not take as they are: the layer runs with zeros behind every
    head's entries, in pages of the larger sizes, and gives the same results; a 32-bit layer runs as it is."""
    cuts = ([300], [268] + [1] * 32, [17] * 17 + [11])
    for sizes, window, rot in (((128, 6, 2, 40, 24), 64, mech.ROTATIONS[1]), ((96, 4, 4, 80, 112), None, mech.ROTATIONS[2]),
                               ((64, 5, 1, 12, 20), 33, mech.ROTATIONS[4])):
        mech.attention_part(DEV, torch.bfloat16, sizes=sizes, window=window, rot=rot, page_size=16, length=300, cuts=cuts, std=0.1)
    part, _, _ = mech._attention_part(DEV, torch.bfloat16, (128, 6, 2, 40, 24), 0.1, 64, None)
    assert (part.run_key_dim, part.run_value_dim) == (64, 32)
    assert (part.cache_need().head_dim, part.cache_need().value_dim) == (64, 32) and (part.key_dim, part.value_dim) == (40, 24)
    part, _, _ = mech._attention_part(DEV, torch.float32, (128, 6, 2, 40, 24), 0.1, 64, None)
    assert (part.run_key_dim, part.run_value_dim) == (40, 24)


@pytest.mark.parametrize("dtype", DTYPES)
def test_window_edges(dtype):
    mech.window_edges(DEV, dtype)
    mech.window_edges(DEV, dtype, page_size=4, window=9, T=60)
    mech.window_edges(DEV, dtype, window=None, T=200)


@pytest.mark.parametrize("sizes", [(64, 8, 2, 64, 64), (64, 4, 2, 96, 112)])
def test_window_edges_on_the_matrix_cores(sizes):
    mech.window_edges(DEV, torch.bfloat16, sizes=sizes, window=64, T=300, std=0.1)
    mech.window_edges(DEV, torch.bfloat16, sizes=sizes, window=129, T=300, std=0.1)
    mech.window_edges(DEV, torch.bfloat16, sizes=sizes, window=None, T=500, std=0.1)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["mixed", "units", "no_loop", "only_recurrent", "aligned"])
def test_cuts_match_plain(tmp_path, name, dtype):
    cases.cuts_match_plain(tmp_path, DEV, name, dtype, length=45 if name != "aligned" else 70)


def test_mistakes_would_show(tmp_path):
    cases.mistakes_would_show(tmp_path, DEV)


@pytest.mark.parametrize("name, dtype", [("mixed", "float32"), ("aligned_dense", "bfloat16")])
def test_layers_match_plain(tmp_path, name, dtype):
    cases.layers_match_plain(tmp_path, DEV, name, dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["mixed", "only_recurrent", "aligned"])
def test_batches_match_alone(tmp_path, name, dtype):
    cases.batches_match_alone(tmp_path, DEV, name, dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_portions_and_pages_of_sixteen(tmp_path, dtype):
    cases.cuts_match_plain(tmp_path, DEV, "aligned", dtype, length=171, page_size=16)
    cases.batches_match_alone(tmp_path / "b", DEV, "aligned", dtype, page_size=16)


@pytest.mark.parametrize("seed", range(12))
def test_drawn_configurations(tmp_path, seed):
    cases.drawn_configuration_runs(tmp_path, DEV, seed)


@pytest.mark.parametrize("seed", [1, 4, 7, 10])
def test_drawn_configurations_bfloat16(tmp_path, seed):
    cases.drawn_configuration_runs(tmp_path, DEV, seed, "bfloat16")


@pytest.mark.parametrize("name, dtype", [("mixed", "float32"), ("aligned", "bfloat16")])
def test_long_decoding(tmp_path, name, dtype):
    cases.long_decoding(tmp_path, DEV, name, dtype, steps=150, page_size=16)


@pytest.mark.parametrize("name, dtype, page_size", [("mixed", "float32", 4), ("mixed", "bfloat16", 4), ("aligned", "bfloat16", 16)])
def test_recorded_decode_steps(tmp_path, name, dtype, page_size):
    """Decode-only steps are recorded in a HIP graph and replayed: three requests decode together for 40 steps, and each
    step's logits are those of the same step run eagerly by a second engine (states advance exactly once)."""
    d = cases.write_model(name, str(tmp_path / "m"))
    V = plain.load(d)[1]["vocab"]
    prompts = {r: cases.random_tokens(n, V, 70 + n) for r, n in (("a", 9), ("b", 3), ("c", 14))}
    follow = {r: cases.random_tokens(40, V, 90 + len(p)) for r, p in prompts.items()}
    engines = [cases.make_executor(d, DEV, dtype, page_size=page_size, num_pages=64, batch=4, max_len=64, graphs=g)
               for g in (True, False)]
    for ex in engines:
        for r, p in prompts.items():
            ex.add_request(r)
        ex.step([StepEntry(r, p, []) for r, p in prompts.items()])
    for k in range(40):
        outs = [ex.step([StepEntry(r, [follow[r][k]], [0]) for r in prompts]).clone() for ex in engines]
        torch.testing.assert_close(outs[0], outs[1], rtol=0, atol=0)


def test_greedy_generation(tmp_path):
    cases.greedy_generation(tmp_path, DEV, "mixed", "float32")


def test_greedy_generation_bfloat16_runs(tmp_path):
    """The serving path as it is used: bfloat16, recorded decode steps, several steps in a row on the device."""
    from simply_amd.engine.llm import LMInterface
    from simply_amd.sampling import SamplingParams

    d = cases.write_model("aligned", str(tmp_path / "m"), dtype=torch.bfloat16)
    lm = LMInterface(d, activation_dtype="bfloat16", batch_size=4, max_seq_len=128, device=DEV)
    prompts = [cases.random_tokens(n, 256, n) for n in (5, 33, 17, 2, 60)]
    outs = lm.generate(prompts, sampling_params=SamplingParams(temperature=0.0, max_decode_steps=24))
    again = lm.generate(prompts, sampling_params=SamplingParams(temperature=0.0, max_decode_steps=24))
    assert all(len(o.output_token_ids) == 24 for o in outs)
    assert [o.output_token_ids for o in outs] == [o.output_token_ids for o in again]


def test_trace_replay_child_process(tmp_path):
    """bin/trace_run as a user starts it: a folder whose config.json leaves the decays' ranks to the tensors, steps on
    standard input, logits in files; two live requests."""
    import json
    import os
    import subprocess

    import numpy as np

    d = cases.write_model("mixed", str(tmp_path / "m"), dtype=torch.bfloat16)
    path = os.path.join(d, "config.json")
    raw = json.load(open(path))
    for l in raw["layers"]:
        l["mixer"].pop("rank", None)
    json.dump(raw, open(path, "w"))
    w, cfg = plain.load(d)
    tx, ty = cases.random_tokens(30, cfg["vocab"], 5), cases.random_tokens(12, cfg["vocab"], 6)
    wx, wy = plain.forward(w, cfg, tx), plain.forward(w, cfg, ty)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": tx[:17], "want": [0, 16]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": tx[17:19], "want": []}, {"id": "y", "tokens": ty[:11], "want": [10]}],
              "end": []},
             {"step": 2, "entries": [{"id": "y", "tokens": ty[11:], "want": [0]}, {"id": "x", "tokens": tx[19:], "want": [10]}],
              "end": ["x", "y"]}]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    out = tmp_path / "out"
    r = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", d, "--dtype", "float32", "--out", str(out),
                        "--max-tokens", "128"], input="\n".join(json.dumps(s) for s in steps) + "\n", text=True,
                       capture_output=True, timeout=600)
    assert r.returncode == 0, r.stderr
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    got = [torch.from_numpy(np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(n, -1)) for i, n in ((0, 2), (1, 1), (2, 2))]
    # (what 32-bit rounding does to this model by itself)
    own = max(float(cases.rel_rows(plain.forward(w, cfg, t, dtype=torch.float32), o).max()) for t, o in ((tx, wx), (ty, wy)))
    for g, want in zip(got, (wx[[0, 16]], wy[[10]], torch.stack([wy[11], wx[29]]))):
        assert float(cases.rel_rows(g, want).max()) <= max(cases.BOUND_F32, 6.0 * own)
