"""Typed configuration of Nozizen, read from the model folder's `config.json`.

A decoder whose layers are listed one by one; a run of consecutive layers may be looped over several times with the same
weights, every pass with a cache and state of its own.  The residual is "streams" parallel streams with learned reads,
writes and mixes around every part (hyper-connections); parts read RMS-normed input.  Mixers: "wkv" (token shift,
data-dependent decay per key channel, a matrix of state per head with a bonus for the current token), "mamba2" (a
state-space recurrence with one decay per head behind a short convolution, its result gated and then normed in groups) and
"attention" (windowed grouped-query attention, values of a size of their own, rotary in half-split pairs on the first
entries of a head, with frequencies scaled by a ramp).  Feed-forward: dense with a squared relu, a mixture of experts
(SiLU-gated; the largest biased logits choose, their softmax among themselves weighs), or none.  The head is the embedding.

Keys: "architecture", "vocab", "width", "streams", "norm": {"eps"}, "embedding": {"scale"}, "layers": [{"type", "mixer":
{...}, "mlp": {...} | null}], "loop": {"start", "stop", "times"}.  wkv: heads, dim (the decay's rank is the first dimension
of the tensor "l<i>.mix.w1"; a config that is to be written with random weights may say it as "rank").  mamba2: heads,
vdim, state, groups, conv, norm_groups.  attention: heads, kv_heads, dim, vdim, scale, optional mask {size}, optional rot
{dims, base, optional scaling {factor, original, fast, slow}}.  mlp: {"kind": "dense", "ff"} or {"kind": "moe", "expert":
{"ff"}, "router": {"experts", "top"}}.
Tensors: "embed", "l<i>.norm1", "l<i>.norm2", "l<i>.hc1.*", "l<i>.hc2.*" (in, mix, out), "l<i>.mix.*", "l<i>.mlp.*",
"final.norm"; matrices are [out, in].
"""
from __future__ import annotations

import copy
import dataclasses
from typing import Any, Mapping

from ..registry import ARCHITECTURES
from .gemma2 import ConfigError
from .nemidra import _positive
from .spec import LayerSpec, ModelSpec, PartSpec, ScheduleEntry
from .zenuzen import _get

LAYER_TYPES = ("wkv", "mamba2", "attention")
MLP_KINDS = ("dense", "moe")


@dataclasses.dataclass(frozen=True)
class NozizenConfig:
    #: the dictionary of config.json, as read (`to_dict` gives it back)
    raw: Mapping[str, Any]
    vocab: int
    width: int
    streams: int
    norm_eps: float
    embedding_scale: float
    num_layers: int
    #: not part of the design: the longest sequence that the engine plans for when --max_seq_len does not say
    max_position: int = 8192
    eos_token_ids: tuple[int, ...] = ()
    initializer_range: float = 0.02

    architecture = "Nozizen"

    @classmethod
    def from_dict(cls, d: Mapping[str, Any], check: bool = True) -> "NozizenConfig":
        layers = _get(d, "layers", "top level")
        if not isinstance(layers, (list, tuple)) or not layers:
            raise ConfigError('config.json: "layers" must be a non-empty list')
        eos = d.get("eos_token_id")
        eos_ids = () if eos is None else tuple(int(e) for e in (eos if isinstance(eos, (list, tuple)) else [eos]))
        eps = _get(_get(d, "norm", "top level"), "eps", "norm", float)
        if eps < 0:
            raise ConfigError("config.json: norm.eps must not be negative")
        cfg = cls(raw=copy.deepcopy(dict(d)), vocab=_positive(_get(d, "vocab", "top level", int), "vocab"),
                  width=_positive(_get(d, "width", "top level", int), "width"),
                  streams=_positive(_get(d, "streams", "top level", int), "streams"), norm_eps=eps,
                  embedding_scale=_get(_get(d, "embedding", "top level"), "scale", "embedding", float),
                  num_layers=len(layers), max_position=int(d.get("max_position", 8192)), eos_token_ids=eos_ids,
                  initializer_range=float(d.get("initializer_range", 0.02)))
        if check:
            cfg.model_spec()   # (reads every key: whatever is missing or wrong is said now)
        return cfg

    @classmethod
    def from_dict_open(cls, d: Mapping[str, Any]) -> "NozizenConfig":
        """The configuration of a model folder before `resolve_shapes` has read the sizes that the tensors give."""
        return cls.from_dict(d, check=False)

    def to_dict(self) -> dict[str, Any]:
        return copy.deepcopy(dict(self.raw))

    def resolve_shapes(self, shapes: Mapping[str, tuple]) -> "NozizenConfig":
        """Sizes that config.json leaves to the tensors: the rank of every wkv mixer's decay projection."""
        raw = copy.deepcopy(dict(self.raw))
        for i, l in enumerate(raw["layers"]):
            name = f"l{i}.mix.w1"
            if l.get("type") == "wkv" and "rank" not in l.get("mixer", {}) and name in shapes:
                l["mixer"]["rank"] = int(shapes[name][0])
        return type(self).from_dict(raw)

    # ------------------------------------------------------------------ schedule
    def schedule(self) -> tuple[ScheduleEntry, ...]:
        n, loop = self.num_layers, self.raw.get("loop")
        if not loop:
            return tuple(ScheduleEntry(i) for i in range(n))
        start, stop, times = (_get(loop, k, "loop", int) for k in ("start", "stop", "times"))
        if not (0 <= start < stop <= n) or times < 1:
            raise ConfigError(f"config.json: loop: layers {start}..{stop - 1} of {n}, {times} times")
        order = list(range(start)) + list(range(start, stop)) * times + list(range(stop, n))
        return tuple(ScheduleEntry(i) for i in order)

    # ------------------------------------------------------------------ parts
    def _mixer(self, i: int, l: Mapping[str, Any]) -> PartSpec:
        D, eps, p, where = self.width, self.norm_eps, f"l{i}.mix.", f"layers[{i}].mixer"
        m = _get(l, "mixer", f"layers[{i}]")

        def size(key: str) -> int:
            return _positive(_get(m, key, where, int), key)

        if l["type"] == "wkv":
            rank = m.get("rank")
            if rank is None:
                raise ConfigError(f"config.json: {where}: the decay's rank is given neither by \"rank\" nor by the tensor "
                                  f"{p}w1 of a model folder")
            tensors = {"mu_" + s: f"{p}mu.{s}" for s in ("r", "k", "v", "g", "w")}
            tensors.update({s + "_proj": p + s for s in ("r", "k", "v", "g", "o")})
            tensors.update(decay_in=p + "w1", decay_out=p + "w2", decay_base=p + "w0", bonus=p + "u", norm=p + "norm")
            return PartSpec("wkv", {"hidden_size": D, "num_heads": size("heads"), "head_dim": size("dim"),
                                    "decay_rank": _positive(int(rank), "rank"), "norm_eps": eps}, tensors)
        heads = size("heads")
        if l["type"] == "mamba2":
            groups, norm_groups, vdim = size("groups"), size("norm_groups"), size("vdim")
            if heads % groups:
                raise ConfigError(f"config.json: {where}: {heads} heads do not split over {groups} groups")
            if heads * vdim % norm_groups:
                raise ConfigError(f"config.json: {where}: {heads * vdim} channels do not split into {norm_groups} norm_groups")
            return PartSpec("state_space", {
                "hidden_size": D, "num_heads": heads, "num_groups": groups, "state_dim": size("state"), "value_dim": vdim,
                "conv_taps": size("conv"), "norm_groups": norm_groups, "norm_eps": eps,
            }, {"in_proj": p + "in", "conv": p + "conv", "conv_bias": p + "conv.b", "dt_bias": p + "dt_bias",
                "a_log": p + "A_log", "skip": p + "D", "norm": p + "norm", "o_proj": p + "o"})
        kv_heads, dim = size("kv_heads"), size("dim")
        if heads % kv_heads:
            raise ConfigError(f"config.json: {where}: heads {heads} is not a multiple of kv_heads {kv_heads}")
        mask, window = m.get("mask"), None
        if mask is not None:
            window = _positive(_get(mask, "size", where + ".mask", int), "mask.size")
        return PartSpec("gated_attention", {
            "hidden_size": D, "num_heads": heads, "num_kv_heads": kv_heads, "key_dim": dim, "value_dim": size("vdim"),
            "scale": _get(m, "scale", where, float), "output_gate": None, "window": window,
            "position_encoding": self._rotation(m.get("rot"), dim, where + ".rot"),
        }, {"q_proj": p + "q", "k_proj": p + "k", "v_proj": p + "v", "o_proj": p + "o"})

    @staticmethod
    def _rotation(rot: "Mapping[str, Any] | None", dim: int, where: str) -> "PartSpec | None":
        if rot is None:
            return None
        dims = _get(rot, "dims", where, int)
        if dims % 2 or not 0 <= dims <= dim:
            raise ConfigError(f"config.json: {where}: dims {dims} must be even and at most dim {dim}")
        base, scaling = _positive(_get(rot, "base", where, float), "rot.base"), rot.get("scaling")
        if scaling is not None:
            keys = ("factor", "original", "fast", "slow")
            scaling = {k: _positive(_get(scaling, k, where + ".scaling", float), "rot.scaling." + k) for k in keys}
            scaling["kind"] = "ramp"
            if base == 1.0:
                raise ConfigError(f"config.json: {where}: a scaling needs a base other than 1")
        if dims == 0:
            return None
        return PartSpec("partial_rope", {"head_dim": dim, "dims": dims, "base": base, "scaling": scaling})

    def _mlp(self, i: int, mlp: Mapping[str, Any]) -> PartSpec:
        D, p, where = self.width, f"l{i}.mlp.", f"layers[{i}].mlp"
        kind = _get(mlp, "kind", where)
        if kind not in MLP_KINDS:
            raise ConfigError(f"config.json: {where}: unknown kind {kind!r}; known: {', '.join(MLP_KINDS)}")
        if kind == "dense":
            return PartSpec("dense", {"hidden_size": D, "intermediate_size": _positive(_get(mlp, "ff", where, int), "ff"),
                                      "activation": "squared_relu"}, {"up_proj": p + "up", "down_proj": p + "down"})
        router, expert = _get(mlp, "router", where), _get(mlp, "expert", where)
        E = _positive(_get(router, "experts", where + ".router", int), "experts")
        top = _positive(_get(router, "top", where + ".router", int), "top")
        if top > E:
            raise ConfigError(f"config.json: {where}.router: top {top} of {E} experts")
        tensors = {"router": p + "router", "router_bias": p + "router.b"}
        for e in range(E):
            tensors.update({f"e{e}.{n}": f"{p}e{e}.{n}" for n in ("gate", "up", "down")})
        return PartSpec("routed_experts", {
            "hidden_size": D, "num_experts": E, "top": top, "router": "chosen_softmax", "router_bias": True,
            "activation": "silu", "expert_size": _positive(_get(expert, "ff", where + ".expert", int), "expert.ff")}, tensors)

    def model_spec(self) -> ModelSpec:
        d, D = self.raw, self.width

        def norm(name: str) -> PartSpec:
            return PartSpec("rmsnorm", {"dim": D, "eps": self.norm_eps, "scale_plus_one": False}, {"scale": name})

        layers, ignorable = [], []
        for i, l in enumerate(d["layers"]):
            p, where = f"l{i}.", f"layers[{i}]"
            kind = _get(l, "type", where)
            if kind not in LAYER_TYPES:
                raise ConfigError(f"config.json: {where}: unknown layer type {kind!r}; known: {', '.join(LAYER_TYPES)}")
            norms, ffn = {"pre_mixer": norm(p + "norm1")}, None
            connections = {f"mixer_{n}": f"{p}hc1.{n}" for n in ("in", "mix", "out")}
            if l.get("mlp") is not None:
                ffn = self._mlp(i, l["mlp"])
                norms["pre_ffn"] = norm(p + "norm2")
                connections.update({f"ffn_{n}": f"{p}hc2.{n}" for n in ("in", "mix", "out")})
            else:
                # (a folder may hold what stands around a feed-forward that is not there)
                ignorable += [p + "norm2"] + [f"{p}hc2.{n}" for n in ("in", "mix", "out")]
            layers.append(LayerSpec(block=PartSpec("hyper_connections", {"streams": self.streams}, connections),
                                    mixer=self._mixer(i, l), feed_forward=ffn, norms=norms))
        spec = ModelSpec(
            architecture=self.architecture, hidden_size=D, vocab_size=self.vocab,
            embedding=PartSpec("scaled_embedding", {"vocab_size": self.vocab, "dim": D, "scale": self.embedding_scale,
                                                    "round_scale": False}, {"table": "embed"}),
            layers=tuple(layers), schedule=self.schedule(), final_norm=norm("final.norm"),
            head=PartSpec("linear_head", {"vocab_size": self.vocab, "dim": D, "soft_cap": None}, {"weight": "embed"}),
            max_position=self.max_position, eos_token_ids=self.eos_token_ids, initializer_range=self.initializer_range,
            ignorable=tuple(ignorable), streams=self.streams)
        spec.validate()
        return spec


ARCHITECTURES.register("Nozizen", NozizenConfig)
