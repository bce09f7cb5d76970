"""Kolorax's mechanisms one by one against the plain implementation's functions (tests/plain_kolorax.py): the kernels, as
bodies that take the module of operations (`simply_amd.kernels.ops` on the GPU, `torch_ops` on the CPU), and the parts of
the framework with weights of the test's own, whole and in portions.  Where random inputs would hide a fault (a far key
among hundreds, a bonus, a limit, the token before a portion), inputs are made so that it shows."""
from __future__ import annotations

import torch

import plain_kolorax as plain
from simply_amd import parts as _parts  # noqa: F401  (registers the parts)
from simply_amd.config.spec import PartSpec
from simply_amd.registry import FEED_FORWARDS, MIXERS, NORMS, PASS_INPUTS
from zenuzen_cases import run_mixer
from zenuzen_mechanisms import close, rand, tol_of

CUTS = ([61], [29] + [1] * 32, [7, 5, 3, 2, 11, 2, 2, 29], [2] * 30 + [1], [1] * 61)


def _meta(counts, slots, starts):
    rows, first = [], 0
    for c, s, p in zip(counts, slots, starts):
        rows.append((s, first, c, p))
        first += c
    return torch.tensor(rows, dtype=torch.int32), first


def _load(part, tensors: dict, dtype, device):
    assert set(tensors) == set(part.param_specs())
    for name, spec in part.param_specs().items():
        assert tuple(tensors[name].shape) == tuple(spec.shape), name
    part.load({n: t.to(dtype).to(device) for n, t in tensors.items()})
    return part


# --------------------------------------------------------------------------- norms and sums
def layer_norm_after_a_sum(o, device, dtype):
    """Rows whose mean is a hundred times their spread (a variance from sums of squares would be lost), widths that are no
    multiple of a wave or a workgroup, a row that is added to every row, nothing added."""
    for T, D in ((5, 7), (3, 100), (4, 320), (3, 1500), (2, 2304), (2, 8000)):
        y, h = rand((T, D), 1, 3.0).to(dtype), (rand((T, D), 2) + 300.0).float()
        w, b = rand((D,), 3).to(dtype), rand((D,), 4).to(dtype)
        res = h.clone().to(device)
        out = o.residual_add_next_norm(y.to(device), res, w.to(device), bias=b.to(device), eps=1e-3, mult=0.37, out_dtype=dtype)
        want = h.double() + 0.37 * y.double()
        close(res, want, 2e-6, "residual")
        close(out, plain.layer_norm(want.float().double(), w.double(), b.double(), 1e-3), max(tol_of(dtype), 2e-4), (T, D))
        small = rand((T, D), 5).float()
        row = rand((D,), 6, 2.0).to(dtype)
        res = small.clone().to(device)
        out = o.residual_add_next_norm(row.to(device).expand(T, -1), res, w.to(device), bias=b.to(device), eps=1e-5, out_dtype=dtype)
        close(res, small.double() + row.double(), 2e-6, "one row added to all")
        close(out, plain.layer_norm(small.double() + row.double(), w.double(), b.double(), 1e-5), tol_of(dtype), (T, D))
        res = small.clone().to(device)
        out = o.residual_add_next_norm(None, res, w.to(device), bias=b.to(device), eps=1e-5, out_dtype=dtype)
        close(res, small, 0.0, "the stream stays")
        close(out, plain.layer_norm(small.double(), w.double(), b.double(), 1e-5), tol_of(dtype), "the norm alone")


def layer_norm_part(device, dtype):
    D = 44
    part = NORMS.build("layernorm", dim=D, eps=1e-4)
    w, b = rand((D,), 1), rand((D,), 2)
    _load(part, {"scale": w, "bias": b}, dtype, device)
    x = rand((6, D), 3, 4.0).float()
    wd, bd = w.to(dtype).double(), b.to(dtype).double()
    close(part.forward(x.to(device), dtype), plain.layer_norm(x.double(), wd, bd, 1e-4), tol_of(dtype), "alone")
    y = rand((6, D), 4).to(dtype)      # a block that norms what a part returns: x += norm(y)
    res = x.clone().to(device)
    nxt = part.add_into(res, y.to(device), part, dtype)
    want = x.double() + plain.layer_norm(y.double(), wd, bd, 1e-4)
    close(res, want, 1e-5, "added")
    close(nxt, plain.layer_norm(want, wd, bd, 1e-4), tol_of(dtype), "and normed again")


def pass_input_part(device, dtype):
    """W [x; x0] + step: x's half before x0's, the pass's own row, the result not rounded to the activation type."""
    D = 40
    part = PASS_INPUTS.build("projected_with_embedding", hidden_size=D, times=3)
    proj, step = rand((D, 2 * D), 1, 0.3), rand((3, D), 2)
    _load(part, {"proj": proj, "step": step}, dtype, device)
    norm = NORMS.build("layernorm", dim=D, eps=1e-5)
    nw, nb = rand((D,), 3), rand((D,), 4)
    _load(norm, {"scale": nw, "bias": nb}, dtype, device)
    w = {"loop.in": proj.to(dtype).double(), "loop.step": step.to(dtype).double()}

    class Ctx:
        pass
    ctx = Ctx()
    ctx.dtype = dtype
    for T in (1, 5, 70):
        x, x0 = rand((T, D), 5).to(dtype).float(), rand((T, D), 6).to(dtype).float()
        for t in range(3):
            want = plain.begin_pass(w, t, x.double(), x0.double())
            h, normed = part.forward(x.clone().to(device), x0.to(device), t, ctx, norm)
            assert h.dtype == torch.float32
            close(h, want, 1e-5, (T, t))     # (32-bit sums of the given operands, in both types)
            close(normed, plain.layer_norm(want, nw.to(dtype).double(), nb.to(dtype).double(), 1e-5), tol_of(dtype), (T, t))
            h, normed = part.forward(x.clone().to(device), x0.to(device), t, ctx, None)
            close(h, want, 1e-5, (T, t))
            assert normed is None


# --------------------------------------------------------------------------- token shift, decays, recurrence
def token_shift(o, device, dtype):
    """Requests of one, two and many tokens in one launch: the first row's predecessor is the slot's tail, and the tail
    moves on to the last row; slots of no request stay; widths with and without 16-byte pieces."""
    for D, streams in ((40, 5), (13, 2), (264, 5), (2056, 1)):
        m, T = _meta([1, 2, 30, 5], [2, 0, 3, 5], [9, 0, 4, 77])
        h = rand((T, D + 16), 1).to(dtype)[:, 8:8 + D]
        mu = rand((streams, D), 2).to(dtype)
        tails = rand((6, D + 12), 3).float()
        dev_tails = tails.clone().to(device)
        got = o.token_shift(h.to(device), mu.to(device), dev_tails[:, 4:4 + D], m.to(device), 4, 30)
        want_tails = tails.clone()
        for slot, first, count, _ in m.tolist():
            hh = h[first:first + count].double()
            before = plain.previous(hh, tails[slot, 4:4 + D].double())
            want = torch.stack([plain.shifted_mix(hh, before, mu[s].double()) for s in range(streams)], 1)
            close(got[first:first + count], want.reshape(count, -1), tol_of(dtype), (D, slot))
            want_tails[slot, 4:4 + D] = hh[-1].float()
        close(dev_tails, want_tails, 0.0, "tails")


def low_rank_decay(o, device, dtype):
    """Ranks below, at and above the pieces that the kernels take; inputs where tanh is nearly linear and where it is
    saturated; decays from nearly 0 to 1 - 1e-4, whose distance from 1 must be right too."""
    from simply_amd.parts.base import as_product_weight

    for T, C, rank in ((5, 36, 3), (33, 64, 32), (70, 130, 64), (20, 48, 71), (1, 16, 16), (300, 4096, 40)):
        p = (rand((T, rank + 5), 1) * torch.tensor([0.003, 0.3, 4.0], dtype=torch.float64)[torch.arange(T) % 3][:, None]).to(dtype)[:, 2:2 + rank]
        w, base = rand((C, rank), 2, 0.5).to(dtype), (rand((C,), 3, 2.0) - 4.0).to(dtype)
        got = o.low_rank_decay(p.to(device), as_product_weight(w.to(device)), base.to(device))
        assert got.dtype == torch.float32
        eye = torch.eye(rank, dtype=torch.float64)
        want = plain.decay(p.double(), eye, w.double(), base.double())
        close(got, want, 3e-6, (T, C, rank))
        log_want, log_got = torch.log(-torch.log(want.clamp(1e-30, 1 - 1e-12))), torch.log(-torch.log(got.double().cpu().clamp(1e-30, 1 - 1e-12)))
        mid = (want > 1e-3) & (want < 1 - 1e-3)
        assert float((log_got - log_want)[mid].abs().max()) < 2e-4, (T, C, rank)   # (one ulp of a near 1 is 6e-8 / 1e-3)


def recurrence_with_bonus(o, device, dtype, sizes=((3, 12), (2, 40), (2, 128), (1, 16), (1, 200), (5, 4), (4, 1), (2, 64))):
    """Requests of 1, 3, 40 and 17 tokens in one launch from states that are not zero; bonuses of both signs; decays near
    0 and near 1; then the same tokens in portions."""
    for H, d in sizes:
        m, T = _meta([1, 3, 40, 17], [1, 3, 0, 2], [9, 0, 4, 30])
        C = H * d
        proj = rand((T, 3 * C + 5), 1, 0.6).to(dtype)
        a = torch.exp(-torch.exp(rand((T, C), 2, 2.0) - 2.0)).float()
        u = rand((C,), 3).to(dtype)
        st = rand((4, C * d + 3), 4, 0.3).float()
        dev_st = st.clone().to(device)
        got = o.linear_state(proj.to(device), 0, C, 2 * C, 1.0, a.to(device), False, H, d, d, False, dev_st, m.to(device), 4,
                             bonus=u.to(device))
        for slot, first, count, _ in m.tolist():
            rows = slice(first, first + count)
            for h in range(H):
                cols = [proj[rows, s * C + h * d:s * C + (h + 1) * d].double() for s in range(3)]
                S0 = st[slot, h * d * d:(h + 1) * d * d].double().view(d, d).T     # kept column by column
                want, S = plain.wkv_recurrence(cols[0], cols[1], cols[2], a[rows, h * d:(h + 1) * d].double(),
                                               u[h * d:(h + 1) * d].double(), S0)
                close(got[rows, h * d:(h + 1) * d], want, 3e-5, (H, d, slot, h))
                close(dev_st[slot, h * d * d:(h + 1) * d * d], S.T.reshape(-1), 3e-5, ("state", H, d, slot, h))
        # one request in portions: the states hand over
        again, at, parts = st.clone().to(device), 0, []
        for n in (1, 2, 16, 17, 3, 1):
            mm = torch.tensor([[0, 0, n, at]], dtype=torch.int32, device=device)
            rows = slice(4 + at, 4 + at + n)
            parts.append(o.linear_state(proj[rows].contiguous().to(device), 0, C, 2 * C, 1.0, a[rows].contiguous().to(device), False, H,
                                        d, d, False, again, mm, 1, bonus=u.to(device)))
            at += n
        close(torch.cat(parts), got[4:44].cpu(), 1e-6, ("portions", H, d))


def head_norm_and_gate(o, device, dtype):
    """Heads to unit RMS, a weight of one entry per head and channel, the gate's silu."""
    T, H, d = 6, 3, 20
    x, g, w = rand((T, H * d), 1, 2.0).float(), rand((T, H * d + 6), 2, 2.0).to(dtype), rand((H * d,), 3).to(dtype)
    gate = g[:, 3:3 + H * d]
    want = plain.rms_unit(x.double().view(T, H, d), 1e-3).reshape(T, -1) * w.double() * plain.silu(gate.double())
    got = o.gated_heads(x.to(device), g.to(device)[:, 3:3 + H * d], H, d, kind=1, weight=w.to(device), eps=1e-3, out_dtype=dtype)
    close(got, want, tol_of(dtype), "a weight per entry")


def wkv_part(device, dtype, sizes=(40, 3, 12, 5), length=61, cuts=CUTS, std=0.3):
    D, H, d, R = sizes
    C = H * d
    p = {"mu." + s: 0.5 + rand((D,), 10 + i, 0.5) for i, s in enumerate("rkvgw")}
    p.update({s: rand((C, D), 20 + i, std) for i, s in enumerate("rkvg")})
    p.update(w1=rand((R, D), 30, std), w2=rand((C, R), 31, 1.0), w0=rand((C,), 32) - 3.0, u=rand((H, d), 33),
             norm=1.0 + rand((C,), 34, 0.3), o=rand((D, C), 35, std))
    part = MIXERS.build("wkv", hidden_size=D, num_heads=H, head_dim=d, decay_rank=R, norm_eps=1e-5)
    names = {"mu_" + s: p["mu." + s] for s in "rkvgw"} | {s + "_proj": p[s] for s in "rkvgo"}
    names |= {"decay_in": p["w1"], "decay_out": p["w2"], "decay_base": p["w0"], "bonus": p["u"], "norm": p["norm"]}
    _load(part, names, dtype, device)
    x = rand((length, D), 40).to(dtype)
    want = plain.wkv({"p." + n: t.to(dtype).double() for n, t in p.items()}, "p.", {"heads": H, "dim": d}, x.double(), 1e-5)
    for c in cuts:
        got = run_mixer(part, x.to(device), c, dtype, device)
        close(got, want, 2e-5 if dtype == torch.float32 else 5e-2, (sizes, c[:4]))


# --------------------------------------------------------------------------- latent attention
def _latent_part(device, dtype, sizes, std, base, dims=None, scale=0.3, alter=None):
    D, H, dk, dr, dv, R = sizes
    dims = dr if dims is None else dims
    m = {"heads": H, "dim": dk, "rot_dim": dr, "vdim": dv, "kv_rank": R, "scale": scale, "rot": {"dims": dims, "base": base}}
    p = {"q": rand((H * (dk + dr), D), 50, std), "dkv": rand((R + dr, D), 51, std), "dkv.norm": 1.0 + rand((R,), 52, 0.3),
         "uk": rand((H * dk, R), 53, std), "uv": rand((H * dv, R), 54, std), "g": rand((H * dv, D), 55, std),
         "o": rand((D, H * dv), 56, std)}
    if alter is not None:
        alter(p)
    part = MIXERS.build("latent_attention", hidden_size=D, num_heads=H, key_dim=dk, rot_dim=dr, value_dim=dv, q_rank=None,
                        kv_rank=R, scale=scale, norm_eps=1e-5, output_gate="element",
                        position_encoding=PartSpec("partial_rope", {"head_dim": dr, "dims": dims, "base": base}))
    _load(part, {"q_proj": p["q"], "dkv_proj": p["dkv"], "dkv_norm": p["dkv.norm"], "uk_proj": p["uk"], "uv_proj": p["uv"],
                 "gate_proj": p["g"], "o_proj": p["o"]}, dtype, device)
    return part, {"p." + n: t.to(dtype).double() for n, t in p.items()}, m


def latent_part(device, dtype, sizes=(40, 3, 12, 8, 10, 24), dims=None, page_size=4, length=61, cuts=CUTS, std=0.3):
    """dims below rot_dim: the rest of the rotated part passes unchanged."""
    part, w, m = _latent_part(device, dtype, sizes, std, 300.0, dims)
    x = rand((length, sizes[0]), 57).to(dtype)
    want = plain.latent_attention(w, "p.", m, x.double(), 1e-5)
    for c in cuts:
        got = run_mixer(part, x.to(device), c, dtype, device, page_size)
        close(got, want, 2e-5 if dtype == torch.float32 else 5e-2, (sizes, dims, c[:4]))


def far_keys(device, dtype, sizes=(40, 3, 12, 8, 10, 24), page_size=16, T=300, std=0.3):
    """One key hundreds of tokens back stands out for one query, through the unrotated part: its score is far above all
    others, so the result is that token's value if it is seen and read from the right place, and something else if not.
    Keys at a page's first and last place and the sequence's first token; the query in a prompt's portion and decoded."""
    D, H, dk, dr, dv, R = sizes

    def alter(p):
        # input channel 0 makes the query's first entry, channel 1 the latent's first entry, which makes the key's first
        p["q"][:, :2] = 0.0
        p["dkv"][:, :2] = 0.0
        p["uk"][:, 0] = 0.0
        for h in range(H):
            p["q"][h * (dk + dr), 0] = 5.0
            p["uk"][h * dk, 0] = 5.0
        p["dkv"][0] = 0.0
        p["dkv"][0, 1] = 6.0

    part, w, m = _latent_part(device, dtype, sizes, std, 10000.0, alter=alter)
    seen = 0.0
    for key in (0, 15, 16, 33, T - 2):
        x = rand((T, D), 58, 0.5)
        x[:, :2] = 0.0
        x[T - 1, 0], x[key, 1] = 6.0, 6.0
        x = x.to(dtype)
        want = plain.latent_attention(w, "p.", m, x.double(), 1e-5)
        without = x.double().clone()
        without[key, 1] = 0.0
        seen = max(seen, float((want - plain.latent_attention(w, "p.", m, without, 1e-5))[-1].abs().max() / want[-1].abs().max()))
        for c in ([T], [T - 1, 1], [T // 3, T // 3, T - 2 * (T // 3) - 1, 1]):
            close(run_mixer(part, x.to(device), c, dtype, device, page_size)[-1:], want[-1:],
                  2e-5 if dtype == torch.float32 else 5e-2, (key, c))
    assert seen > 0.3    # (the made key decides the result)


# --------------------------------------------------------------------------- experts
def clamped_products(o, device, dtype):
    """The gated product with the clamped rule: values on both sides of both limits, at the row counts and sizes that
    different product kernels take."""
    from simply_amd.kernels.packing import pack_gate_up

    for M, N, K in ((3, 20, 24), (5, 48, 64), (40, 48, 64), (70, 96, 128), (300, 256, 192), (1, 16, 40)):
        x = rand((M, K), 1).to(dtype)
        gate, up = rand((N, K), 2, 2.0 / K ** 0.5).to(dtype), rand((N, K), 3, 2.0 / K ** 0.5).to(dtype)
        for limit in (0.7, 3.0):
            g, u = x.double() @ gate.double().T, x.double() @ up.double().T
            assert bool((g > limit).any()) and bool((u.abs() > limit).any() or limit > 1) and bool((g < -limit).any())
            want = plain.clamped_glu(g, u, limit)
            if dtype == torch.bfloat16 and str(device) != "cpu":
                got = o.gemm(x.to(device), pack_gate_up(gate.to(device), up.to(device)), activation=4, limit=limit)
            else:
                got = o.gemm(x.to(device), gate.to(device), w2=up.to(device), activation=4, limit=limit)
            close(got, want, tol_of(dtype), (M, N, K, limit))


def clamped_experts(o, device, dtype):
    """The chosen experts' results, weighted, plus the shared one: rows of few tokens and of many (both tile sizes)."""
    from simply_amd.kernels.packing import stack_experts

    D, F, E, top, limit = 40, 24, 6, 2, 0.8
    mats = {n: [rand(s, 100 * i + e, 0.4).to(dtype) for e in range(E)]
            for i, (n, s) in enumerate((("gate", (F, D)), ("up", (F, D)), ("down", (D, F))))}
    for T in (1, 5, 130):
        x, shared = rand((T, D), 7 + T).to(dtype), rand((T, D), 9).to(dtype)
        g = torch.Generator().manual_seed(T)
        experts = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(T)]).to(torch.int32)
        weights = torch.rand((T, top), generator=g, dtype=torch.float32)
        want = shared.double().clone()
        for t in range(T):
            for k in range(top):
                e = int(experts[t, k])
                w = {"p." + n: mats[n][e].double() for n in mats}
                want[t] += weights[t, k].double() * plain.expert(w, "p.", x[t:t + 1].double(), limit)[0]
        got = o.routed_experts(x.to(device), experts.to(device), weights.to(device),
                               *(stack_experts(m.to(device) for m in mats[n]) for n in ("gate", "up", "down")), 4,
                               shared=shared.to(device), out_dtype=torch.float32, limit=limit)
        close(got, want, 2e-5 if dtype == torch.float32 else 3e-2, f"{T} tokens")


def router_of_groups(o, device, dtype=torch.float32):
    """Softmax scores, groups by their largest score, weights that sum to one: made cases and drawn ones."""
    made = (-3.0 - 0.01 * torch.arange(12, dtype=torch.float64)).expand(2, 12).clone()   # (no two alike)
    made[0, [0, 1, 2]] = torch.tensor([1.0, 0.9, 0.8], dtype=torch.float64)   # group 0: three good ones, none the best
    made[0, 7] = 1.5                                                        # group 2: the best one, the others bad
    made[0, 10] = 1.2                                                       # group 3: the second best
    made[1] = torch.linspace(40.0, -60.0, 12, dtype=torch.float64)          # one score is nearly 1, the others tiny
    cases = [(made, 4, 2, 3), (made, 4, 1, 2), (made, 12, 3, 3), (made, 1, 1, 2)]
    for seed, (E, count, keep, top) in enumerate([(8, 2, 1, 2), (6, 3, 2, 2), (16, 4, 4, 4), (5, 1, 1, 5), (9, 9, 1, 1),
                                                  (64, 8, 3, 6), (130, 1, 1, 3), (4, 4, 4, 4), (512, 16, 5, 70)]):
        cases.append((rand((33, E), 10 + seed, 2.0), count, keep, top))
    for z, count, keep, top in cases:
        z = z.float()
        e, w = o.route_choice(z.to(device), top, 1.0, groups=count, keep=keep, softmax=True, group_best=1, renorm=1e-20)
        e, w = e.cpu().tolist(), w.cpu().double()
        for t in range(z.shape[0]):
            want = dict(plain.choose(z[t].double(), {"top": top, "groups": {"count": count, "keep": keep}}))
            assert sorted(e[t]) == sorted(want), (t, count, keep, top)
            for i, expert in enumerate(e[t]):
                assert abs(float(w[t, i]) - float(want[expert])) < 2e-6, (t, expert)
    # the made row: with two groups of four kept, group 0 stays out although its sum is the largest
    e, _ = o.route_choice(made[:1].float().to(device), 3, 1.0, groups=4, keep=2, softmax=True, group_best=1, renorm=1e-20)
    assert set(e.cpu()[0].tolist()) >= {7, 10} and not set(e.cpu()[0].tolist()) & {0, 1, 2}


def routed_part(device, dtype, experts=6, top=3, groups=(3, 2), ff=24, shared=16, width=40, T=70):
    D = width
    w = {"p.router": rand((experts, D), 1)}
    for e in range(experts):
        w |= {f"p.e{e}.gate": rand((ff, D), 100 + e, 0.3), f"p.e{e}.up": rand((ff, D), 200 + e, 0.3),
              f"p.e{e}.down": rand((D, ff), 300 + e, 0.3)}
    names = {"router": "p.router"} | {f"e{e}.{n}": f"p.e{e}.{n}" for e in range(experts) for n in ("gate", "up", "down")}
    mlp = {"expert": {"ff": ff, "limit": 1.1}, "router": {"experts": experts, "top": top, "groups": {"count": groups[0], "keep": groups[1]}}}
    kw = {}
    if shared:
        w |= {"p.shared.gate": rand((shared, D), 2, 0.3), "p.shared.up": rand((shared, D), 3, 0.3), "p.shared.down": rand((D, shared), 4, 0.3)}
        names |= {f"shared.{n}_proj": f"p.shared.{n}" for n in ("gate", "up", "down")}
        mlp["shared"] = {"ff": shared, "limit": 0.6}
        kw = dict(shared_size=shared, shared_gate=False, shared_limit=0.6)
    part = FEED_FORWARDS.build("routed_experts", hidden_size=D, num_experts=experts, top=top, expert_size=ff, router="softmax",
                               num_groups=groups[0], keep_groups=groups[1], group_score="largest", renormalize=1e-20,
                               activation="clamped_glu", limit=1.1, **kw)
    _load(part, {local: w[name] for local, name in names.items()}, dtype, device)
    x = rand((T, D), 5).to(dtype)
    want = plain.moe({k: v.to(dtype).double() for k, v in w.items()}, "p.", mlp, x.double())
    got = part.forward(x.to(device), None)
    rows = (got.double().cpu() - want).abs().amax(-1) / want.abs().max()
    # (a bfloat16 run may take another expert where two scores are close: a few rows at most)
    tol = 2e-5 if dtype == torch.float32 else 5e-2
    assert int((rows > tol).sum()) <= (0 if dtype == torch.float32 else 3), float(rows.max())
    alone = torch.cat([part.forward(x[t:t + 1].to(device), None) for t in (0, 1, T - 1)])   # (a row does not feel its batch)
    close(alone, got.cpu()[[0, 1, T - 1]], tol, "rows alone")


def experts_refuse_what_does_not_fit():
    import pytest

    for bad in (dict(activation="clamped_glu"), dict(activation="silu", limit=1.0), dict(activation="clamped_glu", limit=0.0),
                dict(activation="clamped_glu", limit=1.0, gated=False), dict(group_score="best")):
        with pytest.raises(ValueError):
            FEED_FORWARDS.build("routed_experts", hidden_size=8, num_experts=4, top=2, expert_size=8, shared_size=8,
                                **({"shared_limit": bad["limit"]} if bad.get("limit") else {}), **bad)


# --------------------------------------------------------------------------- products of several inputs
def products_of_several_inputs(o, device, sizes=((5, 5, 48, 64, 16), (8, 5, 2048, 512, 64), (40, 3, 64, 128, 64), (70, 5, 256, 256, 20),
                                                 (600, 5, 512, 320, 64), (2100, 4, 1024, 512, 1024), (300, 2, 80, 72, 8), (9, 3, 36, 40, 7),
                                                 (130, 3, 32, 20, 32), (700, 5, 208, 64, 3))):
    """Every section against the product of its own; a last section with fewer rows; sizes that the few-rows, the tiled
    and the wide kernels take, and sizes that none takes; rows that are a view."""
    from simply_amd.kernels.ops import SectionedWeight

    for T, S, N, K, last in sizes:
        for dtype in (torch.float32, torch.bfloat16):
            if dtype == torch.float32 and T > 100:
                continue
            ws = [rand((N if s < S - 1 else last, K), s, K ** -0.5).to(dtype) for s in range(S)]
            x = rand((T, S * K + 8), 50).to(dtype)[:, 8:]
            got = o.gemm_sections(x.to(device), SectionedWeight([w.to(device) for w in ws]))
            want = torch.cat([x[:, s * K:(s + 1) * K].double() @ ws[s].double().T for s in range(S)], 1)
            close(got, want, tol_of(dtype), (T, S, N, K, last))


def wide_products_in_32_bit(o, device, sizes=((100, 512, 64), (2048, 1024, 256), (200, 700, 1024), (70, 516, 128))):
    """32-bit results of bfloat16 operands at sizes that the wide kernel takes: not rounded on the way."""
    from simply_amd.parts.base import as_product_weight

    for M, N, K in sizes:
        x, w = rand((M, K), 1).to(torch.bfloat16), rand((N, K), 2, K ** -0.5).to(torch.bfloat16)
        got = o.gemm(x.to(device), as_product_weight(w.to(device)), out_dtype=torch.float32)
        assert got.dtype == torch.float32
        close(got, x.double() @ w.double().T, 2e-5, (M, N, K))


def queries_with_a_gate_per_entry(o, device, dtype):
    T, H, I, O = 7, 3, 20, 12
    x, w, g = rand((T, H * I), 1).to(dtype), rand((H, O, I), 2, 0.3).to(dtype), rand((T, H * O + 5), 3, 2.0).to(dtype)
    for rows in (T, 1):
        gate = g[:rows, 2:2 + H * O]
        want = torch.cat([x[:rows, h * I:(h + 1) * I].double() @ w[h].double().T for h in range(H)], 1) * torch.sigmoid(gate.double())
        close(o.head_product(x[:rows].to(device), w.to(device), gate=g.to(device)[:rows, 2:2 + H * O]), want, tol_of(dtype), rows)
    big = rand((70, H * I), 4).to(dtype)
    gate = rand((70, H * O), 5).to(dtype)
    want = torch.cat([big[:, h * I:(h + 1) * I].double() @ w[h].double().T for h in range(H)], 1) * torch.sigmoid(gate.double())
    close(o.head_product(big.to(device), w.to(device), gate=gate.to(device)), want, tol_of(dtype), "many rows")
