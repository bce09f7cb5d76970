"""Typed configuration of Kolorax, read from the model folder's `config.json`.

A decoder whose layers are listed one by one; a run of consecutive layers may be looped over several times with the same
weights, every pass with a cache and state of its own.  Before every pass (the first too) the stream x becomes
W_in [x; x0] + step_t, with x0 the embedding's output and a learned vector per pass.  A layer is a pre-norm block with a
residual multiplier m, x += m * mixer(norm(x)), x += m * ff(norm(x)), its norms layer norms with weight and bias.  Mixers:
"wkv" (token shift, data-dependent decay per key channel, a matrix of state per head with a bonus for the current token)
and "latent_attention" (keys and values through a normed latent, one rotated key part for all heads, rotary in half-split
pairs, a sigmoid gate per entry).  The feed-forward is a mixture of experts whose two factors are clamped, routed by a
softmax within the best groups of experts, with an optional shared expert, or none.

Keys: "architecture", "vocab", "width", "residual_mult", "norm": {"eps"}, "embedding": {"scale"}, "layers": [{"type",
"mixer": {...}, "mlp": {...} | null}], "loop": {"start", "stop", "times"}.  wkv: heads, dim (the decay's rank is the first
dimension of the tensor "l<i>.mix.w1"; a config that is to be written with random weights may say it as "rank").
latent_attention: heads, dim, rot_dim, vdim, kv_rank, scale, rot {base, dims}.  mlp: {"kind": "moe", "expert": {"ff",
"limit"}, "router": {"experts", "top", "groups": {"count", "keep"}}, "shared": {"ff", "limit"}}.
Tensors: "embed", "loop.in", "loop.step", "l<i>.norm1", "l<i>.norm2" (each with ".b"), "l<i>.mix.*", "l<i>.mlp.*",
"final.norm", "final.norm.b", "head"; matrices are [out, in].
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

LAYER_TYPES = ("wkv", "latent_attention")
MLP_KINDS = ("moe",)
#: the chosen experts' scores are divided by their sum plus this: fixed by the design
WEIGHT_SUM_EPS = 1e-20


@dataclasses.dataclass(frozen=True)
class KoloraxConfig:
    #: the dictionary of config.json, as read (`to_dict` gives it back)
    raw: Mapping[str, Any]
    vocab: int
    width: int
    residual_mult: float
    norm_eps: float
    embedding_scale: float
    num_layers: int
    #: not part of the design: the longest sequence that the engine plans for when --max_seq_len does not say
    max_position: int = 8192
    eos_token_ids: tuple[int, ...] = ()
    initializer_range: float = 0.02

    architecture = "Kolorax"

    @classmethod
    def from_dict(cls, d: Mapping[str, Any], check: bool = True) -> "KoloraxConfig":
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
                  residual_mult=_get(d, "residual_mult", "top level", float), norm_eps=eps,
                  embedding_scale=_get(_get(d, "embedding", "top level"), "scale", "embedding", float),
                  num_layers=len(layers), max_position=int(d.get("max_position", 8192)), eos_token_ids=eos_ids,
                  initializer_range=float(d.get("initializer_range", 0.02)))
        if check:
            cfg.model_spec()   # (reads every key: whatever is missing or wrong is said now)
        return cfg

    @classmethod
    def from_dict_open(cls, d: Mapping[str, Any]) -> "KoloraxConfig":
        """The configuration of a model folder before `resolve_shapes` has read the sizes that the tensors give."""
        return cls.from_dict(d, check=False)

    def to_dict(self) -> dict[str, Any]:
        return copy.deepcopy(dict(self.raw))

    def resolve_shapes(self, shapes: Mapping[str, tuple]) -> "KoloraxConfig":
        """Sizes that config.json leaves to the tensors: the rank of every wkv mixer's decay projection."""
        raw = copy.deepcopy(dict(self.raw))
        for i, l in enumerate(raw["layers"]):
            name = f"l{i}.mix.w1"
            if l.get("type") == "wkv" and "rank" not in l.get("mixer", {}) and name in shapes:
                l["mixer"]["rank"] = int(shapes[name][0])
        return type(self).from_dict(raw)

    # ------------------------------------------------------------------ schedule
    def _loop(self) -> "tuple[int, int, int] | None":
        loop, n = self.raw.get("loop"), self.num_layers
        if not loop:
            return None
        start, stop, times = (_get(loop, k, "loop", int) for k in ("start", "stop", "times"))
        if not (0 <= start < stop <= n) or times < 1:
            raise ConfigError(f"config.json: loop: layers {start}..{stop - 1} of {n}, {times} times")
        return start, stop, times

    def schedule(self) -> tuple[ScheduleEntry, ...]:
        n, loop = self.num_layers, self._loop()
        if loop is None:
            return tuple(ScheduleEntry(i) for i in range(n))
        start, stop, times = loop
        entries = [ScheduleEntry(i) for i in range(start)]
        for t in range(times):
            entries += [ScheduleEntry(i, begins_pass=t if i == start else None) for i in range(start, stop)]
        return tuple(entries + [ScheduleEntry(i) for i in range(stop, n)])

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
        rot_dim, rot = size("rot_dim"), m.get("rot")
        encoding = None
        if rot is not None:
            dims = rot.get("dims", rot_dim)
            if isinstance(dims, bool) or not isinstance(dims, int) or dims % 2 or not 0 <= dims <= rot_dim:
                raise ConfigError(f"config.json: {where}.rot: dims {dims!r} must be even and at most rot_dim {rot_dim}")
            base = _positive(_get(rot, "base", where + ".rot", float), "rot.base")
            encoding = PartSpec("partial_rope", {"head_dim": rot_dim, "dims": dims, "base": base})
        return PartSpec("latent_attention", {
            "hidden_size": D, "num_heads": size("heads"), "key_dim": size("dim"), "rot_dim": rot_dim,
            "value_dim": size("vdim"), "q_rank": None, "kv_rank": size("kv_rank"), "scale": _get(m, "scale", where, float),
            "norm_eps": eps, "output_gate": "element", "position_encoding": encoding,
        }, {"q_proj": p + "q", "dkv_proj": p + "dkv", "dkv_norm": p + "dkv.norm", "uk_proj": p + "uk", "uv_proj": p + "uv",
            "gate_proj": p + "g", "o_proj": p + "o"})

    def _mlp(self, i: int, mlp: Mapping[str, Any]) -> PartSpec:
        D, p, where = self.width, f"l{i}.mlp.", f"layers[{i}].mlp"
        kind = _get(mlp, "kind", where)
        if kind not in MLP_KINDS:
            raise ConfigError(f"config.json: {where}: unknown kind {kind!r}; known: {', '.join(MLP_KINDS)}")
        router, shared, expert = _get(mlp, "router", where), mlp.get("shared"), _get(mlp, "expert", where)
        E = _positive(_get(router, "experts", where + ".router", int), "experts")
        top = _positive(_get(router, "top", where + ".router", int), "top")
        groups = router.get("groups")
        count, keep = (1, 1) if groups is None else (
            _positive(_get(groups, k, where + ".router.groups", int), k) for k in ("count", "keep"))
        if E % count or keep > count or top > keep * (E // count):
            raise ConfigError(f"config.json: {where}.router: {top} of {E} experts in {count} groups of which {keep} stay")
        tensors = {"router": p + "router"}
        for e in range(E):
            tensors.update({f"e{e}.{n}": f"{p}e{e}.{n}" for n in ("gate", "up", "down")})
        params: dict[str, Any] = {
            "hidden_size": D, "num_experts": E, "top": top, "router": "softmax", "num_groups": count, "keep_groups": keep,
            "group_score": "largest", "renormalize": WEIGHT_SUM_EPS, "activation": "clamped_glu",
            "expert_size": _positive(_get(expert, "ff", where + ".expert", int), "expert.ff"),
            "limit": _positive(_get(expert, "limit", where + ".expert", float), "expert.limit")}
        if shared is not None:
            params.update(shared_size=_positive(_get(shared, "ff", where + ".shared", int), "shared.ff"), shared_gate=False,
                          shared_limit=_positive(_get(shared, "limit", where + ".shared", float), "shared.limit"))
            tensors.update({f"shared.{n}_proj": f"{p}shared.{n}" for n in ("gate", "up", "down")})
        return PartSpec("routed_experts", params, tensors)

    def model_spec(self) -> ModelSpec:
        d, D = self.raw, self.width

        def norm(name: str) -> PartSpec:
            return PartSpec("layernorm", {"dim": D, "eps": self.norm_eps}, {"scale": name, "bias": name + ".b"})

        layers, ignorable = [], []
        for i, l in enumerate(d["layers"]):
            p, where = f"l{i}.", f"layers[{i}]"
            kind = _get(l, "type", where)
            if kind not in LAYER_TYPES:
                raise ConfigError(f"config.json: {where}: unknown layer type {kind!r}; known: {', '.join(LAYER_TYPES)}")
            norms, ffn = {"pre_mixer": norm(p + "norm1")}, None
            if l.get("mlp") is not None:
                ffn = self._mlp(i, l["mlp"])
                norms["pre_ffn"] = norm(p + "norm2")
            else:
                ignorable += [p + "norm2", p + "norm2.b"]   # (a folder may hold the norm of a feed-forward that is not there)
            layers.append(LayerSpec(block=PartSpec("pre_norm", {"mult": self.residual_mult}), mixer=self._mixer(i, l),
                                    feed_forward=ffn, norms=norms))
        loop = self._loop()
        spec = ModelSpec(
            architecture=self.architecture, hidden_size=D, vocab_size=self.vocab,
            embedding=PartSpec("scaled_embedding", {"vocab_size": self.vocab, "dim": D, "scale": self.embedding_scale,
                                                    "round_scale": False}, {"table": "embed"}),
            layers=tuple(layers), schedule=self.schedule(), final_norm=norm("final.norm"),
            head=PartSpec("linear_head", {"vocab_size": self.vocab, "dim": D, "soft_cap": None}, {"weight": "head"}),
            max_position=self.max_position, eos_token_ids=self.eos_token_ids, initializer_range=self.initializer_range,
            ignorable=tuple(ignorable),
            pass_input=None if loop is None else PartSpec("projected_with_embedding", {"hidden_size": D, "times": loop[2]},
                                                          {"proj": "loop.in", "step": "loop.step"}))
        spec.validate()
        return spec


ARCHITECTURES.register("Kolorax", KoloraxConfig)
