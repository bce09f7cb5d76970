"""Kolorax without a GPU: configuration and weights, every mechanism's plain torch reference against the plain
implementation's function, and the framework's host logic (model, parts, cache and state manager, the loop over layers,
step function, scheduler) with the kernels replaced by those references."""
import copy
import json
import os

import pytest
import torch

import kolorax_cases as cases
import kolorax_mechanisms as mech
import plain_kolorax as plain
import torch_ops
from simply_amd.config import ConfigError, KoloraxConfig, config_from_dict, load_config
from simply_amd.models import DecoderModel
from simply_amd.weights import WeightsError, load_weights

CPU = "cpu"


# ------------------------------------------------------------------ configuration, registry, weights
def test_config_and_schedule():
    cfg = config_from_dict(cases.MIXED)
    assert isinstance(cfg, KoloraxConfig) and cfg.to_dict() == cases.MIXED
    spec = cfg.model_spec()
    assert [(e.layer, e.begins_pass) for e in spec.schedule] == \
        [(0, None), (1, 0), (2, None), (1, 1), (2, None), (1, 2), (2, None), (3, None)]
    assert [(e.layer, e.begins_pass) for e in config_from_dict(cases.UNITS).model_spec().schedule] == [(0, 0), (1, None), (2, None)]
    assert config_from_dict(cases.NO_LOOP).model_spec().pass_input is None
    model = DecoderModel(spec)
    names = model.expected_tensors()
    assert {"embed", "loop.in", "loop.step", "l0.norm1", "l0.norm1.b", "l0.mix.mu.w", "l0.mix.r", "l0.mix.u", "l1.mix.q", "l1.mix.dkv.norm",
            "l0.mlp.e5.down", "l0.mlp.shared.up", "l2.mlp.router", "final.norm", "final.norm.b", "head"} <= set(names)
    assert names["loop.in"].shape == (40, 80) and names["loop.step"].shape == (3, 40)
    assert names["l1.mix.g"].shape == (30, 40) and names["l0.mix.w2"].shape == (36, 5)
    assert "l3.norm2" not in names and "l1.mlp.shared.gate" not in names and "l1.mix.dq" not in names
    # every pass of the loop has a cache or a state of its own
    needs = model.cache_needs()
    assert len(needs) == len(spec.schedule) and all(c is None for _, c in needs)
    assert needs[0][0].shape == (3 * 12 * 12 + 40,)                         # the heads' matrices, then the last token's h
    assert (needs[1][0].head_dim, needs[1][0].value_dim, needs[1][0].num_kv_heads) == (24 + 8, 24, 1)
    moe = spec.layers[0].feed_forward.params
    assert (moe["limit"], moe["shared_limit"], moe["num_groups"], moe["keep_groups"], moe["top"]) == (1.2, 0.7, 3, 2, 3)


@pytest.mark.parametrize("change, message", [
    (lambda d: d["layers"][0].update(type="conv"), "unknown layer type"),
    (lambda d: d["layers"][0]["mixer"].pop("rank"), "rank"),
    (lambda d: d["layers"][1]["mixer"].pop("scale"), "scale"),
    (lambda d: d["layers"][1]["mixer"]["rot"].update(dims=7), "even"),
    (lambda d: d["layers"][1]["mixer"]["rot"].update(dims=10), "rot_dim"),
    (lambda d: d["layers"][1]["mixer"]["rot"].pop("base"), "base"),
    (lambda d: d["layers"][1]["mlp"].update(kind="dense"), "unknown kind"),
    (lambda d: d["layers"][1]["mlp"]["expert"].pop("limit"), "limit"),
    (lambda d: d["layers"][0]["mlp"]["shared"].update(limit=0.0), "limit"),
    (lambda d: d["layers"][0]["mlp"]["router"]["groups"].update(count=4), "groups"),
    (lambda d: d["layers"][0]["mlp"]["router"].update(top=5), "groups"),
    (lambda d: d["loop"].update(stop=9), "loop"),
    (lambda d: d["loop"].update(times=0), "loop"),
    (lambda d: d.pop("residual_mult"), "residual_mult"),
    (lambda d: d["embedding"].pop("scale"), "scale"),
    (lambda d: d["norm"].pop("eps"), "eps"),
])
def test_config_errors(change, message):
    d = copy.deepcopy(cases.MIXED)
    change(d)
    with pytest.raises(ConfigError, match=message):
        config_from_dict(d)


def test_folder_round_trip_rank_from_the_tensor_and_tolerated_norms(tmp_path):
    """A folder whose config.json does not say the decay's rank: the tensor's shape does.  The norm of a feed-forward that
    a layer does not have may be stored and is left unread; anything else that is unexpected is an error."""
    from safetensors.torch import load_file, save_file

    d = cases.write_model("mixed", str(tmp_path / "m"))
    path = os.path.join(d, "config.json")
    raw = json.load(open(path))
    for l in raw["layers"]:
        l["mixer"].pop("rank", None)
    json.dump(raw, open(path, "w"))
    cfg = load_config(d)
    assert [l.mixer.params.get("decay_rank") for l in cfg.model_spec().layers] == [5, None, 3, None]
    tensors = load_file(os.path.join(d, "model.safetensors"))
    tensors["l3.norm2"], tensors["l3.norm2.b"] = torch.zeros(40), torch.zeros(40)
    save_file(tensors, os.path.join(d, "model.safetensors"))
    load_weights(DecoderModel(cfg.model_spec()), d, torch.float32, torch.device("cpu"))
    tensors["l3.norm3"] = torch.zeros(40)
    del tensors["l0.norm1.b"]
    save_file(tensors, os.path.join(d, "model.safetensors"))
    with pytest.raises(WeightsError) as e:
        load_weights(DecoderModel(cfg.model_spec()), d, torch.float32, torch.device("cpu"))
    assert e.value.missing == ["l0.norm1.b"] and e.value.unexpected == ["l3.norm3"]


def test_embedding_scale_is_not_rounded():
    from simply_amd.registry import EMBEDDINGS

    part = EMBEDDINGS.build(**{"name": "scaled_embedding"}, vocab_size=4, dim=3, scale=1.303, round_scale=False)
    assert part.scale == 1.303 and not part.round_scale
    spec = config_from_dict(dict(cases.MIXED, embedding={"scale": 1.303})).model_spec()
    assert spec.embedding.params["scale"] == 1.303 and spec.embedding.params["round_scale"] is False


# ------------------------------------------------------------------ the plain implementation's own invariants
def test_plain_recurrence_in_portions_and_without_a_state():
    r, k, v, a = (mech.rand((12, 5), i) for i in range(4))
    a, u = torch.sigmoid(a), mech.rand((5,), 9)
    whole, S = plain.wkv_recurrence(r, k, v, a, u)
    first, S1 = plain.wkv_recurrence(r[:5], k[:5], v[:5], a[:5], u)
    second, S2 = plain.wkv_recurrence(r[5:], k[5:], v[5:], a[5:], u, S1)
    torch.testing.assert_close(torch.cat([first, second]), whole)
    torch.testing.assert_close(S2, S)
    torch.testing.assert_close(whole[0], (r[0] * u * k[0]).sum() * v[0])      # only the bonus reads the first token
    torch.testing.assert_close(whole[1], (r[1] * u * k[1]).sum() * v[1] + (r[1] * k[0]).sum() * v[0])   # the decay comes later


def test_plain_latent_attention_is_the_one_with_absorbed_products():
    """Rotations in half-split pairs depend on the distance of two positions alone."""
    q, k = mech.rand((1, 8), 1).expand(30, 8), mech.rand((1, 8), 2).expand(30, 8)
    pos = torch.arange(30)
    s = plain.rotate_half(q, pos, 6, 50.0) @ plain.rotate_half(k, pos, 6, 50.0).T
    torch.testing.assert_close(s[20, 13], s[9, 2])
    assert float((s[20, 13] - s[20, 14]).abs()) > 1e-3


# ------------------------------------------------------------------ the references of the kernels, one by one
@pytest.mark.parametrize("body", [mech.layer_norm_after_a_sum, mech.token_shift, mech.low_rank_decay, mech.recurrence_with_bonus,
                                  mech.head_norm_and_gate, mech.clamped_products, mech.clamped_experts, mech.router_of_groups,
                                  mech.queries_with_a_gate_per_entry])
def test_reference_of_a_kernel(body):
    body(torch_ops, CPU, torch.float32)


def test_reference_of_products_of_several_inputs():
    mech.products_of_several_inputs(torch_ops, CPU, sizes=((5, 5, 48, 64, 16), (9, 3, 36, 40, 7)))


@pytest.mark.parametrize("body", [mech.layer_norm_part, mech.pass_input_part, mech.wkv_part, mech.latent_part, mech.routed_part])
def test_part(cpu_ops, body):
    body(CPU, torch.float32)


def test_parts_at_other_sizes(cpu_ops):
    mech.wkv_part(CPU, torch.float32, sizes=(24, 1, 4, 9), length=9, cuts=([9], [2, 2, 2, 2, 1], [1] * 9))   # a rank above the heads
    mech.latent_part(CPU, torch.float32, sizes=(24, 2, 4, 6, 5, 8), dims=4, length=12, cuts=([12], [5, 2, 5], [1] * 12))
    mech.routed_part(CPU, torch.float32, experts=4, top=4, groups=(1, 1), shared=None, T=9)
    mech.experts_refuse_what_does_not_fit()


def test_far_keys(cpu_ops):
    mech.far_keys(CPU, torch.float32, T=120)


# ------------------------------------------------------------------ the engine's host logic
@pytest.mark.parametrize("name", ["units", "no_loop", "only_wkv"])
def test_cuts_match_plain(tmp_path, cpu_ops, name):
    cases.cuts_match_plain(tmp_path, CPU, name)


def test_cuts_match_plain_and_mistakes_would_show(tmp_path, cpu_ops):
    cases.mistakes_would_show(tmp_path, CPU)


@pytest.mark.parametrize("name", ["mixed", "only_wkv"])
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
