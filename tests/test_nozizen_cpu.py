"""Nozizen without a GPU: configuration and weights, every mechanism's plain torch reference against the plain
implementation's function, and the framework's host logic (model, parts, cache and state manager, the loop over layers,
step function, scheduler) with the kernels replaced by those references."""
import copy
import json
import os

import pytest
import torch

import nozizen_cases as cases
import nozizen_mechanisms as mech
import plain_nozizen as plain
import torch_ops
from simply_amd.config import ConfigError, NozizenConfig, config_from_dict, load_config
from simply_amd.models import DecoderModel
from simply_amd.weights import WeightsError, load_weights

CPU = "cpu"


# ------------------------------------------------------------------ configuration, registry, weights
def test_config_and_schedule():
    cfg = config_from_dict(cases.MIXED)
    assert isinstance(cfg, NozizenConfig) and cfg.to_dict() == cases.MIXED
    spec = cfg.model_spec()
    assert [e.layer for e in spec.schedule] == [0, 1, 2, 1, 2, 1, 2, 3] == plain.schedule(cases.MIXED)
    assert [e.layer for e in config_from_dict(cases.NO_LOOP).model_spec().schedule] == [0, 1, 2, 3]
    model = DecoderModel(spec)
    names = model.expected_tensors()
    assert {"embed", "l0.norm1", "l0.hc1.in", "l0.hc2.mix", "l0.mix.mu.w", "l0.mix.u", "l1.mix.in", "l1.mix.conv.b", "l1.mix.A_log",
            "l1.mix.D", "l2.mix.q", "l1.mlp.router.b", "l1.mlp.e5.down", "l0.mlp.up", "final.norm"} <= set(names)
    assert names["l1.mix.in"].shape == (40 + 40 + 2 * 2 * 12 + 4, 40) and names["l1.mix.conv"].shape == (88, 3)
    assert names["l0.hc1.mix"].shape == (3, 3) and names["l2.mix.o"].shape == (40, 84)
    assert "head" not in names and "l3.norm2" not in names and "l3.hc2.in" not in names
    # every pass of the loop has a cache or a state of its own
    needs = model.cache_needs()
    assert len(needs) == len(spec.schedule) and all(c is None for _, c in needs)
    assert needs[0][0].shape == (3 * 12 * 12 + 40,)
    assert needs[1][0].shape == (4 * 10 * 12 + 2 * 88,)                      # the heads' states, then the convolution's inputs
    assert (needs[2][0].head_dim, needs[2][0].value_dim, needs[2][0].num_kv_heads, needs[2][0].window) == (10, 14, 2, 9)


@pytest.mark.parametrize("change, message", [
    (lambda d: d["layers"][0].update(type="conv"), "unknown layer type"),
    (lambda d: d["layers"][0]["mixer"].pop("rank"), "rank"),
    (lambda d: d["layers"][1]["mixer"].pop("state"), "state"),
    (lambda d: d["layers"][1]["mixer"].update(groups=3), "groups"),
    (lambda d: d["layers"][1]["mixer"].update(norm_groups=7), "norm_groups"),
    (lambda d: d["layers"][1]["mixer"].update(conv=0), "conv"),
    (lambda d: d["layers"][2]["mixer"].pop("scale"), "scale"),
    (lambda d: d["layers"][2]["mixer"].update(kv_heads=4), "kv_heads"),
    (lambda d: d["layers"][2]["mixer"]["mask"].update(size=0), "mask.size"),
    (lambda d: d["layers"][2]["mixer"]["rot"].update(dims=7), "even"),
    (lambda d: d["layers"][2]["mixer"]["rot"].update(dims=12), "dim"),
    (lambda d: d["layers"][2]["mixer"]["rot"]["scaling"].pop("fast"), "fast"),
    (lambda d: d["layers"][2]["mixer"]["rot"]["scaling"].update(factor=-1.0), "factor"),
    (lambda d: d["layers"][2]["mlp"].update(kind="sparse"), "unknown kind"),
    (lambda d: d["layers"][0]["mlp"].pop("ff"), "ff"),
    (lambda d: d["layers"][1]["mlp"]["router"].update(top=7), "top"),
    (lambda d: d["layers"][1]["mlp"].pop("expert"), "expert"),
    (lambda d: d["loop"].update(stop=9), "loop"),
    (lambda d: d["loop"].update(times=0), "loop"),
    (lambda d: d.pop("streams"), "streams"),
    (lambda d: d.update(streams=0), "streams"),
    (lambda d: d["embedding"].pop("scale"), "scale"),
    (lambda d: d["norm"].pop("eps"), "eps"),
])
def test_config_errors(change, message):
    d = copy.deepcopy(cases.MIXED)
    change(d)
    with pytest.raises(ConfigError, match=message):
        config_from_dict(d)


def test_folder_round_trip_rank_from_the_tensor_and_tolerated_tensors(tmp_path):
    """A folder whose config.json does not say the decay's rank: the tensor's shape does.  What stands around a feed-forward
    that a layer does not have may be stored and is left unread; anything else that is unexpected is an error."""
    from safetensors.torch import load_file, save_file

    d = cases.write_model("mixed", str(tmp_path / "m"))
    path = os.path.join(d, "config.json")
    raw = json.load(open(path))
    for l in raw["layers"]:
        l["mixer"].pop("rank", None)
    json.dump(raw, open(path, "w"))
    cfg = load_config(d)
    assert [l.mixer.params.get("decay_rank") for l in cfg.model_spec().layers] == [5, None, None, None]
    tensors = load_file(os.path.join(d, "model.safetensors"))
    tensors["l3.norm2"], tensors["l3.hc2.in"] = torch.zeros(40), torch.zeros(3)
    save_file(tensors, os.path.join(d, "model.safetensors"))
    load_weights(DecoderModel(cfg.model_spec()), d, torch.float32, torch.device("cpu"))
    tensors["l3.norm3"] = torch.zeros(40)
    del tensors["l0.hc1.out"]
    save_file(tensors, os.path.join(d, "model.safetensors"))
    with pytest.raises(WeightsError) as e:
        load_weights(DecoderModel(cfg.model_spec()), d, torch.float32, torch.device("cpu"))
    assert e.value.missing == ["l0.hc1.out"] and e.value.unexpected == ["l3.norm3"]


def test_streams_go_with_blocks_of_as_many_and_with_no_other_schedule():
    import dataclasses

    spec = config_from_dict(cases.MIXED).model_spec()
    for change in (dict(streams=2), dict(streams=None),
                   dict(schedule=tuple(dataclasses.replace(e, add_embedding=True) for e in spec.schedule))):
        with pytest.raises(ValueError, match="stream"):
            dataclasses.replace(spec, **change).validate()


# ------------------------------------------------------------------ the plain implementation's own invariants
def test_plain_recurrence_in_portions():
    x, B, C = (mech.rand((12, n), i) for i, n in enumerate((3, 5, 5)))
    dt, a, d = plain.softplus(mech.rand((12,), 3)), torch.tensor(0.3, dtype=torch.float64), torch.tensor(0.7, dtype=torch.float64)
    whole, S = plain.ssd_recurrence(x, B, C, dt, a, d)
    first, S1 = plain.ssd_recurrence(x[:5], B[:5], C[:5], dt[:5], a, d)
    second, S2 = plain.ssd_recurrence(x[5:], B[5:], C[5:], dt[5:], a, d, S1)
    torch.testing.assert_close(torch.cat([first, second]), whole)
    torch.testing.assert_close(S2, S)
    torch.testing.assert_close(whole[0], dt[0] * (B[0] @ C[0]) * x[0] + 0.7 * x[0])      # (the token reads its own update)


def test_plain_streams():
    """Equal streams with rows of a mix that sum to one and no result written stay equal; the mix is [from, to]."""
    x = mech.rand((4, 1, 6), 1).expand(-1, 3, -1)
    mix = torch.softmax(mech.rand((3, 3), 2), 0)
    out = plain.write_streams(x, mix, torch.zeros(3, dtype=torch.float64), mech.rand((4, 6), 3))
    torch.testing.assert_close(out, x)
    one = torch.zeros(1, 2, 1, dtype=torch.float64)
    one[0, 0] = 1.0
    moved = plain.write_streams(one, torch.tensor([[0.0, 2.0], [5.0, 0.0]], dtype=torch.float64), torch.zeros(2, dtype=torch.float64),
                                torch.zeros(1, 1, dtype=torch.float64))
    assert moved.flatten().tolist() == [0.0, 2.0]


def test_plain_reference_of_the_recurrence():
    mech.plain_recurrence_is_the_one_of_the_logarithms()


def test_scaled_frequencies():
    mech.scaled_frequencies()


# ------------------------------------------------------------------ the references of the kernels, one by one
@pytest.mark.parametrize("body", [mech.streams, mech.convolution_and_gates, mech.group_norm_behind_a_gate, mech.rotated_inputs,
                                  mech.router_among_the_chosen])
def test_reference_of_a_kernel(body):
    body(torch_ops, CPU, torch.float32)


@pytest.mark.parametrize("pieces", [False, True])
def test_reference_of_the_recurrence(pieces):
    mech.recurrence_of_groups(torch_ops, CPU, torch.float32, pieces)
    mech.far_token_in_the_recurrence(torch_ops, CPU, torch.float32, pieces)


@pytest.mark.parametrize("body", [mech.streams_block, mech.state_space_part, mech.wkv_part, mech.attention_part, mech.routed_part,
                                  mech.dense_part])
def test_part(cpu_ops, body):
    body(CPU, torch.float32)


def test_parts_at_other_sizes(cpu_ops):
    mech.state_space_part(CPU, torch.float32, sizes=(24, 1, 1, 1, 1, 1, 1), length=9, cuts=([9], [2, 2, 2, 2, 1], [1] * 9))
    mech.state_space_part(CPU, torch.float32, sizes=(24, 6, 3, 4, 8, 8, 2), length=40, cuts=([40], [2, 13, 2, 23], [1] * 40))
    mech.attention_part(CPU, torch.float32, sizes=(24, 3, 3, 4, 4), window=1, rot=None, length=12, cuts=([12], [5, 2, 5], [1] * 12))
    mech.attention_part(CPU, torch.float32, sizes=(24, 4, 1, 8, 2), window=None, rot=mech.ROTATIONS[3], length=30, cuts=([30], [1] * 30))
    mech.routed_part(CPU, torch.float32, experts=4, top=4, T=9)
    mech.parts_refuse_what_does_not_fit()


def test_window_edges(cpu_ops):
    mech.window_edges(CPU, torch.float32, T=80)
    mech.window_edges(CPU, torch.float32, window=None, T=80)


# ------------------------------------------------------------------ the engine's host logic
@pytest.mark.parametrize("name", ["units", "no_loop", "only_recurrent"])
def test_cuts_match_plain(tmp_path, cpu_ops, name):
    cases.cuts_match_plain(tmp_path, CPU, name)


def test_cuts_match_plain_and_mistakes_would_show(tmp_path, cpu_ops):
    cases.mistakes_would_show(tmp_path, CPU)


@pytest.mark.parametrize("name", ["mixed", "only_recurrent"])
def test_batches_match_alone(tmp_path, cpu_ops, name):
    cases.batches_match_alone(tmp_path, CPU, name)


@pytest.mark.parametrize("seed", range(5))
def test_drawn_configurations(tmp_path, cpu_ops, seed):
    cases.drawn_configuration_runs(tmp_path, CPU, seed)


def test_layers_match_plain(tmp_path, cpu_ops):
    cases.layers_match_plain(tmp_path, CPU)


def test_long_decoding(tmp_path, cpu_ops):
    cases.long_decoding(tmp_path, CPU, "mixed", steps=60, page_size=4)


def test_greedy_generation(tmp_path, cpu_ops):
    cases.greedy_generation(tmp_path, CPU)
