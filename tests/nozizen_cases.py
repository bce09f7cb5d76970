"""Small Nozizen configurations, model folders with random weights, and the bodies of the tests that run the framework
against the plain implementation (tests/plain_nozizen.py).  A body takes the device; the CPU tests run it with the kernels
replaced by their plain torch references (the `cpu_ops` fixture), the GPU tests with the kernels themselves."""
from __future__ import annotations

import copy
import os

import torch

import plain_nozizen as plain
from simply_amd.config import config_from_dict
from simply_amd.engine import StepEntry
from simply_amd.weights import write_random_model
from zenuzen_cases import make_executor, random_tokens, run_cut  # noqa: F401  (shared helpers)


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def wkv(heads, dim, rank, mlp=None):
    return {"type": "wkv", "mixer": {"heads": heads, "dim": dim, "rank": rank}, "mlp": mlp}


def mamba2(heads, groups, vdim, state, conv, norm_groups, mlp=None):
    return {"type": "mamba2", "mlp": mlp, "mixer": {"heads": heads, "groups": groups, "vdim": vdim, "state": state, "conv": conv,
                                                    "norm_groups": norm_groups}}


def attention(heads, kv_heads, dim, vdim, scale, window=None, rot=None, scaling=None, mlp=None):
    """rot: (dims, base); scaling: (factor, original, fast, slow)."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if window:
        m["mask"] = {"size": window}
    if rot:
        m["rot"] = {"dims": rot[0], "base": rot[1]}
        if scaling:
            m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return {"type": "attention", "mixer": m, "mlp": mlp}


def config(vocab, width, streams, eps, scale, layers, loop=None):
    d = {"architecture": "Nozizen", "vocab": vocab, "width": width, "streams": streams, "norm": {"eps": eps},
         "embedding": {"scale": scale}, "layers": layers}
    if loop:
        d["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return d


#: odd sizes everywhere; three streams; a loop over the two middle layers, three times, with a kind of layer each; values
#: larger than keys, rotation on a part of a head with scaled frequencies; norm groups that do not follow the heads
MIXED = config(83, 40, 3, 1e-5, 2.5, [
    wkv(3, 12, 5, mlp=dense(28)),
    mamba2(4, 2, 10, 12, 3, 5, mlp=moe(6, 3, 24)),
    attention(6, 2, 10, 14, 0.35, window=9, rot=(6, 500.0), scaling=(4.0, 64, 8.0, 1.0), mlp=moe(5, 1, 12)),
    mamba2(3, 3, 8, 5, 5, 1),
], loop=(1, 3, 3))
#: what the others make unequal is equal or 1 here: one stream, one head of one or a few entries, one tap, a window of the
#: token itself, every expert used, one group, a loop that runs once over everything, a decay whose rank is above the heads
UNITS = config(31, 24, 1, 1e-6, 1.0, [
    wkv(1, 4, 7, mlp=moe(3, 3, 8)),
    mamba2(1, 1, 1, 1, 1, 1, mlp=dense(8)),
    attention(1, 1, 4, 4, 0.5, window=1, rot=(2, 10.0), scaling=(1.0, 16, 1.0, 1.0), mlp=moe(4, 1, 8)),
    mamba2(4, 4, 4, 4, 2, 4),
    attention(2, 1, 4, 2, 0.5, window=2),
], loop=(0, 5, 1))
#: no loop, no window, no rotation; two streams
NO_LOOP = config(40, 32, 2, 1e-5, 0.7, [attention(4, 4, 8, 8, 0.3, mlp=moe(4, 2, 16)),
                                        mamba2(2, 1, 16, 8, 4, 2, mlp=dense(32)), attention(4, 1, 8, 12, 0.3, rot=(8, 100.0)),
                                        wkv(2, 16, 4)])
#: only recurrent layers, looped twice from the start; five streams; width no multiple of 8
ONLY_RECURRENT = config(53, 30, 5, 1e-4, 2.0, [mamba2(6, 3, 6, 9, 8, 3, mlp=moe(2, 1, 12)), wkv(3, 8, 6, mlp=dense(20))],
                        loop=(0, 1, 2))
#: sizes in multiples of 16, 32 and 64 (what fast kernels may take), still small; windows that portions and decoded tokens
#: run past
ALIGNED = config(256, 128, 4, 1e-5, 1.5, [
    wkv(2, 64, 32, mlp=moe(8, 2, 64)),
    mamba2(4, 2, 32, 64, 4, 2, mlp=dense(256)),
    attention(8, 2, 64, 64, 0.1, window=40, rot=(32, 20000.0), scaling=(8.0, 256, 16.0, 1.0), mlp=moe(4, 2, 128)),
    mamba2(8, 1, 48, 128, 4, 4),
    attention(8, 4, 96, 64, 0.12, window=21, rot=(96, 1000.0), mlp=dense(128)),
], loop=(1, 3, 2))
#: the same without experts: no row can take another one, so that in bfloat16 too every layer can be held to a bound
ALIGNED_DENSE = dict(ALIGNED, layers=[dict(l, mlp=dense(128)) for l in ALIGNED["layers"]])
#: name -> (configuration, seed, standard deviation of the matrices, of the norms' weights and biases)
CONFIGS = {"mixed": (MIXED, 41, 0.25, 0.3), "units": (UNITS, 42, 0.25, 0.3), "no_loop": (NO_LOOP, 43, 0.25, 0.3),
           "only_recurrent": (ONLY_RECURRENT, 44, 0.25, 0.3), "aligned": (ALIGNED, 45, 0.1, 0.2),
           "aligned_dense": (ALIGNED_DENSE, 46, 0.1, 0.2)}


def drawn_config(seed: int) -> dict:
    """A configuration drawn at random: streams, sizes, head counts, groups, the order of the layers, windows, rotations,
    feed-forwards, the loop, eps."""
    import random

    r = random.Random(900 + seed)

    def mlp():
        x = r.random()
        if x < 0.2:
            return None
        if x < 0.55:
            return dense(r.choice([8, 20, 36]))
        E = r.randint(1, 7)
        return moe(E, r.randint(1, min(E, 4)), r.choice([8, 20, 36]))

    layers = []
    for _ in range(r.randint(2, 5)):
        kind = r.random()
        if kind < 0.25:
            layers.append(wkv(r.choice([1, 2, 3]), r.choice([4, 8, 16, 40]), r.choice([1, 2, 6, 16]), mlp=mlp()))
        elif kind < 0.65:
            groups, per = r.choice([1, 2, 3]), r.choice([1, 2, 3])
            vdim = r.choice([4, 6, 8, 20, 32])
            parts = [n for n in range(1, 9) if groups * per * vdim % n == 0]
            layers.append(mamba2(groups * per, groups, vdim, r.choice([4, 8, 12, 24, 72]), r.choice([1, 2, 3, 4, 6]),
                                 r.choice(parts), mlp=mlp()))
        else:
            kv, per, dim = r.choice([1, 2, 3]), r.choice([1, 2, 3, 4]), r.choice([4, 8, 12, 24])
            rot = r.choice([None, (dim, 50.0), (dim // 2, 10000.0)])
            scaling = r.choice([None, (2.0, 32, 4.0, 1.0), (8.0, 4096, 32.0, 1.0)])
            layers.append(attention(kv * per, kv, dim, r.choice([4, 8, 20]), r.choice([0.2, 0.4]), window=r.choice([None, 3, 8, 17]),
                                    rot=rot, scaling=scaling, mlp=mlp()))
    n, loop = len(layers), None
    if r.random() < 0.75:
        start = r.randrange(n)
        loop = (start, r.randint(start + 1, n), r.randint(1, 3))
    return config(r.choice([50, 97, 130]), r.choice([24, 40, 56, 64, 100]), r.choice([1, 2, 3, 4, 6]), r.choice([1e-6, 1e-5, 1e-3]),
                  r.choice([0.5, 1.0, 4.0]), layers, loop=loop)


def write_folder(d: dict, seed: int, out_dir: str, dtype, std: float, norm_std: float) -> str:
    """The configuration with random weights through the framework's random-weights mode; then the norms' weights are
    moved to around one, the decays' constants to half-lives of about a dozen tokens (a state that is lost or taken from
    another request shows for long), and the streams' weights to where every stream is read, mixed and written."""
    from safetensors.torch import load_file, save_file

    folder = write_random_model(config_from_dict(d), out_dir, seed, torch.float32, std=std, norm_std=norm_std)
    path = os.path.join(folder, "model.safetensors")
    tensors = load_file(path)
    S = d["streams"]
    for name, t in tensors.items():
        if name.endswith(("norm", "norm1", "norm2", ".hc1.out", ".hc2.out", "mix.D")):
            t += 1.0
        elif name.endswith((".hc1.in", ".hc2.in")):
            t += 1.0 / S
        elif name.endswith((".hc1.mix", ".hc2.mix")):
            t += 0.6 * torch.eye(S) + 0.2 / S
        elif name.endswith("mix.w0"):
            t -= 3.0
        elif name.endswith("mix.dt_bias"):
            t -= 1.5
        elif name.endswith("mix.A_log"):
            t *= 3.0
            t -= 1.0
        elif ".mix.mu." in name:
            t += 0.5
        elif name.endswith("mix.conv"):
            t += 0.4
        elif name.endswith("router.b"):
            t *= 4.0
    save_file({n: t.to(dtype).contiguous() for n, t in tensors.items()}, path, metadata={"format": "pt"})
    return folder


def write_model(name: str, out_dir: str, dtype=torch.float32, std: float | None = None) -> str:
    d, seed, own_std, norm_std = CONFIGS[name]
    return write_folder(d, seed, out_dir, dtype, std or own_std, norm_std)


def plain_weights(model_dir, dtype):
    """The folder's weights as the engine holds them: a bfloat16 run rounds them first."""
    w, cfg = plain.load(model_dir)
    if dtype == "bfloat16":
        w = {k: (v.to(torch.bfloat16) if v.is_floating_point() else v) for k, v in w.items()}
    return w, cfg


def rel_rows(got: torch.Tensor, want: torch.Tensor) -> torch.Tensor:
    """Every row's error (root mean square over the vocabulary) relative to the logits' root mean square."""
    got, want = got.double().cpu(), want.double().cpu()
    return (got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()


def rounded_run(model_dir: str, tokens) -> torch.Tensor:
    """The logits of the whole sequence from the framework's host logic with the kernels' plain torch references in
    bfloat16, on the CPU: what the roundings alone do to this model on these tokens."""
    import pytest

    import torch_ops
    from simply_amd.kernels import ops

    with pytest.MonkeyPatch.context() as mp:
        for name in torch_ops.STAND_INS:
            mp.setattr(ops, name, getattr(torch_ops, name))
        ex = make_executor(model_dir, "cpu", "bfloat16", page_size=16)
        return run_cut(ex, "r", tokens, [len(tokens)])


#: 32-bit: every row within the bound.  bfloat16: these tiny models with their few experts amplify rounding, and a row
#: whose router is close takes another expert, which moves it and, through the states, some rows behind it; a run that
#: is further off than the first figures is held against what the roundings alone do (`rounded_run`)
BOUND_F32, MEDIAN_BF16, FAR_BF16 = 5e-5, 3e-2, 0.2


def assert_engine_close(got, want, dtype: str, w, cfg, tokens, what=None, model_dir=None) -> None:
    rows = rel_rows(got, want)
    assert torch.isfinite(got).all(), what
    if dtype == "float32":
        own = rel_rows(plain.forward(w, cfg, tokens, dtype=torch.float32), want)
        assert float(rows.max()) <= max(BOUND_F32, 6.0 * float(own.max())), (what, float(rows.max()), float(own.max()))
        return
    far = int((rows > FAR_BF16).sum())
    if float(rows.median()) <= MEDIAN_BF16 and far <= len(rows) // 20:
        return
    own = rel_rows(rounded_run(model_dir, tokens), want)
    own_far = int((own > FAR_BF16).sum())
    assert float(rows.median()) <= max(MEDIAN_BF16, 1.5 * float(own.median())) and far <= max(len(rows) // 20, 2 * own_far + 2), \
        (what, float(rows.median()), float(own.median()), far, own_far, len(rows))


# --------------------------------------------------------------------------- bodies


def cuts_match_plain(tmp_path, device, name, dtype="float32", length=45, page_size=4):
    """Whole prompts, a prompt and then token by token, portions of several sizes down to two tokens, all tokens one by
    one: the same logits.  The first tokens of a sequence are among the wanted places every time."""
    d = write_model(name, str(tmp_path / name))
    w, cfg = plain_weights(d, dtype)
    tokens = random_tokens(length, cfg["vocab"], 7)
    want = plain.forward(w, cfg, tokens)
    ex = make_executor(d, device, dtype, page_size=page_size)
    n = length
    for cuts in ([n], [n - 32] + [1] * 32, [7, 5, 3, 2, 11, 2, 2, n - 32], [2] * (n // 2) + [1] * (n % 2), [1] * n):
        got = run_cut(ex, "r", tokens, cuts)
        assert_engine_close(got, want, dtype, w, cfg, tokens, (name, cuts), d)
    return got, want, w, cfg, tokens


def _zeroed(*ends):
    def mistake(w, cfg):
        return {k: (torch.zeros_like(v) if k.endswith(ends) else v) for k, v in w.items()}, cfg
    mistake.__name__ = "without_" + "_".join(ends)
    return mistake


def _mixers(cfg, kind, change):
    cfg = copy.deepcopy(cfg)
    for l in cfg["layers"]:
        if l["type"] == kind:
            change(l["mixer"])
    return cfg


def _streams_mixed_the_other_way(w, cfg):
    return {k: (v.T.contiguous() if k.endswith(".mix") and ".hc" in k else v) for k, v in w.items()}, cfg


def _window_one_wider(w, cfg):
    return w, _mixers(cfg, "attention", lambda m: m["mask"].update(size=m["mask"]["size"] + 1))


def _window_one_narrower(w, cfg):
    return w, _mixers(cfg, "attention", lambda m: m["mask"].update(size=m["mask"]["size"] - 1))


def _frequencies_not_scaled(w, cfg):
    return w, _mixers(cfg, "attention", lambda m: m["rot"].pop("scaling"))


def _not_rotated(w, cfg):
    return w, _mixers(cfg, "attention", lambda m: m.pop("rot"))


def _normed_as_one_group(w, cfg):
    return w, _mixers(cfg, "mamba2", lambda m: m.update(norm_groups=1))


def _one_expert_fewer(w, cfg):
    cfg = copy.deepcopy(cfg)
    for l in cfg["layers"]:
        router = (l.get("mlp") or {}).get("router")
        if router and router["top"] > 1:
            router["top"] -= 1
    return w, cfg


def _one_pass_fewer(w, cfg):
    cfg = copy.deepcopy(cfg)
    cfg["loop"]["times"] -= 1
    return w, cfg


#: mistakes planted in the plain implementation, each far outside the bound that the engine is held to
MISTAKES = (_zeroed("mix.u"), _zeroed("mix.mu.r", "mix.mu.k", "mix.mu.v", "mix.mu.g", "mix.mu.w"), _zeroed("mix.D"),
            _zeroed("mix.conv.b"), _zeroed("mix.dt_bias"), _zeroed("router.b"), _streams_mixed_the_other_way, _window_one_wider,
            _window_one_narrower, _frequencies_not_scaled, _not_rotated, _normed_as_one_group, _one_expert_fewer,
            _one_pass_fewer)


def mistakes_would_show(tmp_path, device, name="mixed", dtype="float32"):
    got, want, w, cfg, tokens = cuts_match_plain(tmp_path, device, name, dtype)
    for mistake in MISTAKES:
        off = plain.forward(*mistake(w, cfg), tokens)
        assert float(rel_rows(got, off).max()) > 100 * BOUND_F32, mistake.__name__


def run_schedule(ex, schedule, toks, want, dtype, w, cfg, what, model_dir):
    done = {r: 0 for r in toks}
    got = {r: [] for r in toks}
    for step in schedule:
        entries = []
        for r, n in step:
            if not ex.has_request(r):
                ex.add_request(r)
            entries.append(StepEntry(r, toks[r][done[r]:done[r] + n], list(range(n))))
        logits = ex.step(entries).cpu()
        at = 0
        for r, n in step:
            got[r].append(logits[at:at + n])
            at += n
            done[r] += n
            if done[r] == len(toks[r]):
                ex.finish_request(r)
        ex.cache.check()
    for r in toks:
        assert done[r] == len(toks[r])
        if len(toks[r]) >= 20 or dtype == "float32":   # (the typical row of a dozen is no measure)
            assert_engine_close(torch.cat(got[r]), want[r], dtype, w, cfg, toks[r], (what, r), model_dir)


def batches_match_alone(tmp_path, device, name, dtype="float32", page_size=4):
    """Requests of unequal length run together, portions beside single tokens, in a pool so tight that pages and state
    slots are given back and used again (freed pages are filled with NaN; a state slot keeps what its last owner left
    until the next admission), requests that wait for some steps: each request's logits are those of the request alone."""
    d = write_model(name, str(tmp_path / name))
    w, cfg = plain_weights(d, dtype)
    lengths = {"a": 37, "b": 9, "c": 1, "d": 22, "e": 30, "f": 2, "g": 17}
    toks = {r: random_tokens(n, cfg["vocab"], 100 + i) for i, (r, n) in enumerate(lengths.items())}
    want = {r: plain.forward(w, cfg, t) for r, t in toks.items()}
    ex = make_executor(d, device, dtype, page_size=page_size, num_pages=26 if page_size == 4 else 8, batch=3, max_len=48,
                       poison=True)
    run_schedule(ex, [
        [("a", 11), ("b", 3), ("c", 1)],          # c ends: its slot goes to d
        [("a", 2), ("b", 1), ("d", 5)],
        [("a", 1), ("b", 5), ("d", 1)],           # b ends
        [("a", 16), ("d", 2), ("e", 7)],
        [("a", 1), ("d", 1), ("e", 2)],
        [("d", 13), ("e", 1), ("a", 6)],          # a and d end
        [("e", 20), ("f", 2), ("g", 1)],          # e and f end
        [("g", 2)], [("g", 14)],
    ], toks, want, dtype, w, cfg, name, d)


def drawn_configuration_runs(tmp_path, device, seed: int, dtype="float32"):
    """A drawn configuration, three requests of unequal length in portions beside single tokens, in a tight pool."""
    d = write_folder(drawn_config(seed), seed, str(tmp_path / f"m{seed}"), torch.float32, 0.3, 0.3)
    w, cfg = plain_weights(d, dtype)
    toks = {r: random_tokens(n, cfg["vocab"], seed * 10 + i) for i, (r, n) in enumerate((("a", 41), ("b", 13), ("c", 26)))}
    want = {r: plain.forward(w, cfg, t) for r, t in toks.items()}
    ex = make_executor(d, device, dtype, page_size=4, num_pages=24, batch=2, max_len=44, poison=True)
    run_schedule(ex, [[("a", 9), ("b", 2)], [("a", 1), ("b", 7)], [("a", 17), ("b", 1)], [("a", 2), ("b", 3)],   # b ends
                      [("a", 1), ("c", 20)], [("a", 11), ("c", 1)], [("c", 2)], [("c", 3)]], toks, want, dtype, w, cfg, seed, d)


def long_decoding(tmp_path, device, name, dtype="float32", prompt=5, steps=150, page_size=16):
    """A short prompt, then many tokens one by one: states and caches are carried over page and window borders."""
    d = write_model(name, str(tmp_path / name))
    w, cfg = plain_weights(d, dtype)
    tokens = random_tokens(prompt + steps, cfg["vocab"], 21)
    want = plain.forward(w, cfg, tokens)
    ex = make_executor(d, device, dtype, page_size=page_size, num_pages=-(-(prompt + steps) // page_size) + 1)
    got = run_cut(ex, "r", tokens, [prompt] + [1] * steps)
    assert_engine_close(got, want, dtype, w, cfg, tokens, name, d)


def layers_match_plain(tmp_path, device, name="mixed", dtype="float32"):
    """The streams' sum behind every layer run (a looped layer counts each time) against the plain implementation's."""
    d = write_model(name, str(tmp_path / name))
    w, cfg = plain_weights(d, dtype)
    tokens = random_tokens(23, cfg["vocab"], 5)
    want: list = []
    plain.forward(w, cfg, tokens, layers_out=want)
    own: list = []       # (what 32-bit rounding does to this model by itself)
    plain.forward(w, cfg, tokens, dtype=torch.float32, layers_out=own)
    ex = make_executor(d, device, dtype)
    ex.add_request("r")
    T, R, ctx, rows, wants, _ = ex._prepare([StepEntry("r", tokens, [len(tokens) - 1])])
    got: list = []
    ex.model.forward(ex._dev[:T], ctx, ex.cache.views, rows, after_layer=lambda i, h: got.append(h.double().cpu().clone()))
    assert len(got) == len(want) == len(ex.model.spec.schedule)
    for i, (g, x) in enumerate(zip(got, want)):
        err = (g - x).abs().amax(-1) / x.abs().max()
        # (in bfloat16 the typical row: some are amplified further)
        bound = max(2e-5, 6.0 * float((own[i].double() - x).abs().max() / x.abs().max())) if dtype == "float32" else 4e-2
        assert float(err.max() if dtype == "float32" else err.median()) < bound, (i, err)


def greedy_generation(tmp_path, device, name="mixed", dtype="float32"):
    """Greedy generation through the framework's own entry point and scheduler: the plain implementation's tokens."""
    from simply_amd.engine.llm import LMInterface
    from simply_amd.sampling import SamplingParams

    d = write_model(name, str(tmp_path / name), std=0.4)
    w, cfg = plain.load(d)
    prompts = [random_tokens(n, cfg["vocab"], 50 + n) for n in (5, 11, 17, 3)]
    want = [plain.greedy(w, cfg, p, 6) for p in prompts]
    lm = LMInterface(d, activation_dtype=dtype, batch_size=3, max_seq_len=64, page_size=4, max_num_issue_tokens=16,
                     device=str(device))
    outs = lm.generate(prompts, sampling_params=SamplingParams(temperature=0.0, max_decode_steps=6))
    assert [o.output_token_ids for o in outs] == want
