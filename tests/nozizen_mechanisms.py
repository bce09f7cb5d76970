"""Nozizen's mechanisms one by one against the plain implementation's functions (tests/plain_nozizen.py): the kernels, as
bodies that take the module of operations (`simply_amd.kernels.ops` on the GPU, `torch_ops` on the CPU), and the parts of
the framework with weights of the test's own, whole and in portions.  Where random inputs would hide a fault (a key just
inside or outside a window, a token many pieces back in a recurrence, the inputs before a portion), inputs are made so that
it shows."""
from __future__ import annotations

import torch

import plain_nozizen as plain
from kolorax_mechanisms import CUTS, _load, _meta
from simply_amd import parts as _parts  # noqa: F401  (registers the parts)
from simply_amd.config.spec import PartSpec
from simply_amd.registry import BLOCKS, FEED_FORWARDS, MIXERS, NORMS, POSITION_ENCODINGS
from zenuzen_cases import run_mixer
from zenuzen_mechanisms import close, rand, tol_of


# --------------------------------------------------------------------------- streams
def streams(o, device, dtype):
    """The update with the read behind it, the update alone, reads alone (of some rows, without a norm), from separate
    streams and from one row that stands for all; stream counts and widths with and without 16-byte pieces."""
    for T, S, D in ((3, 4, 64), (5, 2, 1032), (2, 4, 2304), (3, 3, 40), (4, 1, 13), (2, 16, 7), (2, 5, 300), (2, 4, 5000),
                    (300, 4, 4096), (2, 4, 4096), (2, 2, 66)):
        x, y = rand((T, S, D), 1).float(), rand((T, D), 2, 2.0).to(dtype)
        mix, ow, iw = rand((S, S), 3).float(), rand((S,), 4).float(), rand((S,), 5).float()
        w = rand((D,), 6).to(dtype)
        dev = [t.to(device) for t in (mix, ow, iw)]
        new = plain.write_streams(x.double(), mix.double(), ow.double(), y.double())
        read = plain.rms_norm(plain.read_streams(new, iw.double()), w.double(), 1e-3)
        h = x.clone().to(device)
        got, z = o.streams(h, y=y.to(device), mix=dev[0], out_weights=dev[1], in_weights=dev[2], weight=w.to(device), eps=1e-3,
                           out_dtype=dtype)
        assert got.data_ptr() == h.data_ptr() and z.dtype == dtype     # (in place)
        close(got, new, 2e-6, ("streams", T, S, D))
        close(z, read, tol_of(dtype), ("read", T, S, D))
        h = x.clone().to(device)
        got, z = o.streams(h, y=y.to(device), mix=dev[0], out_weights=dev[1], out_dtype=dtype)
        close(got, new, 2e-6, ("update alone", T, S, D))
        assert z is None
        # one row that stands for all streams: it is left as it is, the streams get memory of their own
        row = rand((T, D), 7).float().to(device)
        same = row.unsqueeze(1).expand(-1, S, -1)
        kept = row.clone()
        new = plain.write_streams(same.double().cpu(), mix.double(), ow.double(), y.double())
        got, z = o.streams(same, y=y.to(device), mix=dev[0], out_weights=dev[1], in_weights=dev[2], weight=w.to(device), eps=1e-3,
                           out_dtype=dtype)
        close(got, new, 2e-6, ("from one row", T, S, D))
        if S > 1:
            close(row, kept, 0.0, "the row stays")
        close(z, plain.rms_norm(plain.read_streams(new, iw.double()), w.double(), 1e-3), tol_of(dtype), ("from one row", T, S, D))
        # reads alone
        rows = torch.tensor([T - 1, 0, T - 1], dtype=torch.int32)
        u = plain.read_streams(x.double(), iw.double())
        h = x.clone().to(device)
        close(o.streams(h, in_weights=dev[2], weight=w.to(device), eps=1e-3, rows=rows.to(device), out_dtype=dtype)[1],
              plain.rms_norm(u, w.double(), 1e-3)[rows.long()], tol_of(dtype), ("rows", T, S, D))
        close(o.streams(h, in_weights=dev[2])[1], u, 2e-6, ("no norm", T, S, D))
        close(h, x, 0.0, "a read writes nothing")


def streams_from_partial_sums(o, device):
    """A product whose cuts of K are not added up yet, handed to the update as it is."""
    from simply_amd.parts.base import as_product_weight

    seen = 0
    for T, D, K, S in ((8, 2048, 8192, 4), (5, 512, 4096, 3), (200, 1024, 4096, 4), (64, 256, 4096, 2)):
        a, wt = rand((T, K), 1).to(torch.bfloat16), rand((D, K), 2, K ** -0.5).to(torch.bfloat16)
        y = o.gemm(a.to(device), as_product_weight(wt.to(device)), defer_sum=True)
        seen += hasattr(y, "planes")
        x, mix, ow = rand((T, S, D), 3).float(), rand((S, S), 4).float(), rand((S,), 5).float()
        got, _ = o.streams(x.clone().to(device), y=y, mix=mix.to(device), out_weights=ow.to(device), out_dtype=torch.bfloat16)
        want = plain.write_streams(x.double(), mix.double(), ow.double(), a.double() @ wt.double().T)
        close(got, want, 5e-3, (T, D, K, S))
    assert seen


def streams_block(device, dtype):
    """The block around parts that are simple functions: reads, mixes and writes of both sublayers, with and without a
    feed-forward, one block behind another."""
    D, S = 40, 3

    class Doubled:
        defers_sum = False

        def forward(self, x, ctx, *cache):
            return x * 2

    class Shifted:
        defers_sum = False

        def forward(self, x, ctx):
            return x - 0.5

    class Ctx:
        pass
    ctx = Ctx()
    ctx.dtype = dtype
    tensors, blocks = {}, []
    for i, ffn in enumerate((Shifted(), None)):
        norms = {}
        for j, q in enumerate(("pre_mixer", "pre_ffn")[:2 if ffn else 1]):
            norms[q] = NORMS.build("rmsnorm", dim=D, eps=1e-4, scale_plus_one=False)
            tensors[f"l{i}.norm{j + 1}"] = 1.0 + rand((D,), 10 * i + j, 0.3)
            _load(norms[q], {"scale": tensors[f"l{i}.norm{j + 1}"]}, dtype, device)
        block = BLOCKS.build("hyper_connections", Doubled(), ffn, norms, streams=S)
        names = {}
        for j, q in enumerate(("mixer", "ffn")[:2 if ffn else 1]):
            for n, shape in (("in", (S,)), ("mix", (S, S)), ("out", (S,))):
                tensors[f"l{i}.hc{j + 1}.{n}"] = rand(shape, 100 + 10 * i + j, 0.5) + 0.3
                names[f"{q}_{n}"] = tensors[f"l{i}.hc{j + 1}.{n}"]
        _load(block, names, dtype, device)
        blocks.append(block)
    w = {k: v.to(dtype).double() for k, v in tensors.items()}
    x = rand((7, D), 50).float()
    want = torch.stack([x.double()] * S, 1)
    want = plain.sublayer(w, "l0.", 1, want, lambda h: h * 2, 1e-4)
    want = plain.sublayer(w, "l0.", 2, want, lambda h: h - 0.5, 1e-4)
    want = plain.sublayer(w, "l1.", 1, want, lambda h: h * 2, 1e-4)
    h = x.to(device).unsqueeze(1).expand(-1, S, -1)
    h, normed = blocks[0].forward(h, ctx, None, None, blocks[1].first_norm())
    h, normed = blocks[1].forward(h, ctx, None, normed, None)
    assert normed is None
    close(h, want, 5e-6 if dtype == torch.float32 else 2e-2, "two blocks")


# --------------------------------------------------------------------------- state-space recurrence
def convolution_and_gates(o, device, dtype):
    """Requests of 1, 2, 30 and 9 tokens in one launch, slots of no request stay; tap counts from one to eight, shorter
    and longer than a request's tokens; channels with and without pieces of eight; step sizes from tiny to large, whose
    decays' logarithms must be right too; then the same tokens in portions."""
    for C, H, n, at in ((24, 3, 4, 16), (13, 2, 3, 5), (40, 5, 1, 8), (16, 4, 8, 0), (520, 1, 2, 8), (1032, 6, 4, 24), (7, 1, 5, 3)):
        m, T = _meta([1, 2, 30, 9], [2, 0, 3, 5], [9, 0, 4, 77])
        width = -(-(at + C + H) // 8) * 8
        proj = rand((T, width), 1, 1.5).to(dtype)
        taps, bias = rand((C, n), 2).to(dtype), rand((C,), 3).to(dtype)
        dt_bias, a_log = (rand((H,), 4, 4.0) - 3.0).to(dtype), rand((H,), 5, 2.0).to(dtype)
        pad = (-C * (n - 1)) % 4
        tails = rand((6, (n - 1) * C + 4 + pad), 6).float()
        run = lambda rows, tl, mm, s, q: o.ssm_inputs(rows.to(device), at, at + C, C, H, taps.t().contiguous().to(device),  # noqa: E731
                                                      bias.to(device), dt_bias.to(device), a_log.to(device), tl, mm.to(device), s, q)
        dev_tails = tails.clone().to(device)
        y, gates = run(proj, dev_tails[:, 4:], m, 4, 30)
        assert y.dtype == dtype and gates.dtype == torch.float32
        want_tails = tails.clone()
        for slot, first, count, _ in m.tolist():
            x = proj[first:first + count, at:at + C].double()
            old = tails[slot, 4:4 + (n - 1) * C].double().view(n - 1, C)
            close(y[first:first + count], plain.causal_conv(x, taps.double(), bias.double(), old), tol_of(dtype), (C, n, slot))
            want_tails[slot, 4:4 + (n - 1) * C] = torch.cat([old, x])[count:].reshape(-1).float()
        close(dev_tails, want_tails, 0.0, ("tails", C, n))
        dt = plain.softplus(proj[:, at + C:at + C + H].double() + dt_bias.double())
        log_decay = -torch.exp(a_log.double()) * dt
        got = gates.double().cpu()
        assert float((got[:, H:2 * H] / dt - 1).abs().max()) < 1e-5
        assert float((got[:, 2 * H:] / log_decay - 1).abs().max()) < 1e-5
        close(got[:, :H], torch.exp(log_decay), 1e-5, ("decays", C, n))
        again, done, parts = tails.clone().to(device), 0, []
        for k in (1, 2, 9, 17, 1):
            mm = torch.tensor([[3, 0, k, done]], dtype=torch.int32)
            parts.append(run(proj[3 + done:3 + done + k].contiguous(), again[:, 4:], mm, 1, k)[0])
            done += k
        close(torch.cat(parts), y[3:33].cpu(), 1e-6 if dtype == torch.float32 else 5e-3, ("portions", C, n))
        close(again[3], dev_tails[3].cpu(), 0.0, ("tails of portions", C, n))


def group_norm_behind_a_gate(o, device, dtype):
    for T, width, groups in ((5, 24, 3), (3, 20, 1), (2, 39, 13), (4, 1024, 2), (2, 3000, 1), (2, 2048, 8), (1, 6000, 2), (2, 1100, 1)):
        y, z, w = rand((T, width), 1, 3.0).float(), rand((T, width + 8), 2, 2.0).to(dtype), rand((width,), 3).to(dtype)
        want = plain.gated_group_norm(y.double(), z[:, 8:].double(), groups, w.double(), 1e-3)
        got = o.gated_group_norm(y.to(device), z.to(device)[:, 8:], groups, w.to(device), 1e-3)
        assert got.dtype == dtype
        close(got, want, tol_of(dtype), (T, width, groups))


def _recurrence_case(H, G, N, dv, counts, dtype, seed=1, decay=1.0):
    C = H * dv + 2 * G * N
    T = sum(counts)
    proj = rand((T, -(-C // 8) * 8), seed, 0.7).to(dtype)
    dt = torch.nn.functional.softplus(rand((T, H), seed + 1) - 1.0)
    log_decay = -torch.exp(rand((H,), seed + 2)) * dt * decay
    gates = torch.cat([torch.exp(log_decay), dt, log_decay], 1).float()
    return proj, gates, rand((H,), seed + 3).to(dtype), dt.float().double(), log_decay


def _recurrence_wanted(proj, gates, skip, H, G, N, dv, S0):
    """One request's rows: (y [T, H dv], the states [H][dv][N])."""
    inner = H * dv
    y, states = [], []
    for h in range(H):
        g = h // (H // G)
        x = proj[:, h * dv:(h + 1) * dv].double()
        B = proj[:, inner + g * N:inner + (g + 1) * N].double()
        C = proj[:, inner + (G + g) * N:inner + (G + g + 1) * N].double()
        dt = gates[:, H + h].double()
        # (decays from their stored logarithms, which the plain function would compute itself)
        S, out = S0[h].T.clone(), []
        for t in range(x.shape[0]):
            S = torch.exp(gates[t, 2 * H + h].double()) * S + dt[t] * torch.outer(B[t], x[t])
            out.append(S.T @ C[t] + skip[h].double() * x[t])
        y.append(torch.stack(out))
        states.append(S.T)
    return torch.cat(y, 1), torch.stack(states)


def recurrence_of_groups(o, device, dtype, pieces=False):
    """Heads that share queries and keys in groups, a skip, from states that are not zero: requests of 1, 3, 70 and 130
    tokens in one launch, then one of them in portions; decays from nearly none to nearly everything.  pieces: the kernel
    that takes 64 tokens at a time, otherwise token by token."""
    sizes = ((4, 2, 8, 4), (6, 2, 48, 20), (2, 1, 128, 32), (4, 4, 64, 16), (3, 3, 16, 8), (4, 1, 24, 48)) if pieces else \
        ((4, 2, 8, 6), (6, 3, 5, 7), (2, 1, 128, 20), (3, 3, 16, 1), (2, 2, 1, 3), (4, 1, 200, 8))
    for H, G, N, dv in sizes:
        for decay in (0.003, 1.0, 40.0):
            counts = [1, 3, 70, 130] if decay == 1.0 else [1, 90]
            m, T = _meta(counts, [1, 3, 0, 2][:len(counts)], [9, 0, 4, 30][:len(counts)])
            proj, gates, skip, _, _ = _recurrence_case(H, G, N, dv, counts, dtype, decay=decay)
            at = (H * dv + G * N, H * dv, 0)
            st = rand((4, H * N * dv + 4), 9, 0.5).float()
            dev_st = st.clone().to(device)
            if pieces:
                assert o.state_chunks_takes(proj.to(device), *at, N, dv, dev_st)

            def run(rows, gt, state, meta, n):
                if pieces:
                    return o.state_chunks(rows.to(device), *at, gt.to(device), H, G, N, dv, state, meta.to(device), n, skip=skip.to(device))
                return o.linear_state(rows.to(device), *at, 1.0, gt.to(device), True, H, N, dv, False, state, meta.to(device), n,
                                      key_heads=G, skip=skip.to(device))

            got = run(proj, gates, dev_st, m, len(counts))
            wanted = {}
            for slot, first, count, _ in m.tolist():
                S0 = st[slot, :H * N * dv].double().view(H, dv, N)
                want, S = _recurrence_wanted(proj[first:first + count], gates[first:first + count], skip, H, G, N, dv, S0)
                wanted[slot] = want
                close(got[first:first + count], want, 3e-5, (H, G, N, dv, decay, slot))
                close(dev_st[slot, :H * N * dv], S.reshape(-1), 3e-5, ("state", H, G, N, dv, decay, slot))
            close(dev_st[:, H * N * dv:], st[:, H * N * dv:], 0.0, "what lies behind the state")
            slot, first, count, _ = m.tolist()[-1]
            again, done, parts = st.clone().to(device), 0, []
            for n in (2, 17, 64, 1, count - 84):
                mm = torch.tensor([[slot, 0, n, done]], dtype=torch.int32)
                rows = slice(first + done, first + done + n)
                parts.append(run(proj[rows].contiguous(), gates[rows].contiguous(), again, mm, 1))
                done += n
            close(torch.cat(parts), wanted[slot], 3e-5, ("portions", H, G, N, dv, decay))


def plain_recurrence_is_the_one_of_the_logarithms():
    """The reference of the two bodies above against the plain implementation's own function."""
    H, G, N, dv = 4, 2, 5, 3
    proj, gates, skip, dt, log_decay = _recurrence_case(H, G, N, dv, [20], torch.float32)
    a_log = torch.log(-log_decay / dt)
    want, _ = _recurrence_wanted(proj, gates, skip, H, G, N, dv, torch.zeros(H, dv, N, dtype=torch.float64))
    for h in range(H):
        g = h // 2
        y, _ = plain.ssd_recurrence(proj[:, h * dv:(h + 1) * dv].double(), proj[:, H * dv + g * N:H * dv + (g + 1) * N].double(),
                                    proj[:, H * dv + (G + g) * N:H * dv + (G + g + 1) * N].double(), dt[:, h], a_log[0, h],
                                    skip[h].double())
        close(y, want[:, h * dv:(h + 1) * dv], 1e-6, h)


def far_token_in_the_recurrence(o, device, dtype, pieces):
    """With hardly any decay one token's outer product, hundreds of tokens back, decides what one query reads: the token at
    the edges of the pieces, the query at the end."""
    H, G, N, dv, T = 2, 1, 16, 8, 300
    for key in (0, 63, 64, 127, 250, 298):
        proj, gates, skip, _, _ = _recurrence_case(H, G, N, dv, [T], dtype, decay=1e-4)
        proj[:, H * dv] = 0.0                       # key channel 0 belongs to one token
        proj[key, H * dv] = 8.0
        proj[T - 1, H * dv + G * N:H * dv + 2 * G * N] = 0.0
        proj[T - 1, H * dv + G * N] = 8.0           # and to one query
        want, _ = _recurrence_wanted(proj, gates, skip * 0, H, G, N, dv, torch.zeros(H, dv, N, dtype=torch.float64))
        st = torch.zeros((1, H * N * dv), dtype=torch.float32, device=device)
        at, m = (H * dv + G * N, H * dv, 0), torch.tensor([[0, 0, T, 0]], dtype=torch.int32, device=device)
        if pieces:
            got = o.state_chunks(proj.to(device), *at, gates.to(device), H, G, N, dv, st, m, 1)
        else:
            got = o.linear_state(proj.to(device), *at, 1.0, gates.to(device), True, H, N, dv, False, st, m, 1, key_heads=G)
        assert float(want[-1].abs().max()) > 0.5
        close(got[-1:], want[-1:], 3e-5, key)


def state_space_part(device, dtype, sizes=(40, 4, 2, 10, 12, 3, 5), length=61, cuts=CUTS, std=0.3):
    D, H, G, dv, N, taps, parts = sizes
    inner, C = H * dv, H * dv + 2 * G * N
    p = {"in": rand((inner + C + H, D), 1, std), "conv": 0.4 + rand((C, taps), 2, 0.5), "conv.b": rand((C,), 3, 0.3),
         "dt_bias": rand((H,), 4) - 1.5, "A_log": rand((H,), 5) - 1.0, "D": 1.0 + rand((H,), 6, 0.3),
         "norm": 1.0 + rand((inner,), 7, 0.3), "o": rand((D, inner), 8, std)}
    part = MIXERS.build("state_space", hidden_size=D, num_heads=H, num_groups=G, state_dim=N, value_dim=dv, conv_taps=taps,
                        norm_groups=parts, norm_eps=1e-5)
    names = {"in_proj": "in", "conv": "conv", "conv_bias": "conv.b", "dt_bias": "dt_bias", "a_log": "A_log", "skip": "D", "norm": "norm",
             "o_proj": "o"}
    _load(part, {local: p[n] for local, n in names.items()}, dtype, device)
    x = rand((length, D), 40).to(dtype)
    m = {"heads": H, "groups": G, "vdim": dv, "state": N, "conv": taps, "norm_groups": parts}
    want = plain.mamba2({"p." + n: t.to(dtype).double() for n, t in p.items()}, "p.", m, x.double(), 1e-5)
    for c in cuts:
        got = run_mixer(part, x.to(device), c, dtype, device)
        close(got, want, 2e-5 if dtype == torch.float32 else 5e-2, (sizes, c[:4]))


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


# --------------------------------------------------------------------------- rotation, attention
ROTATIONS = (dict(dims=16, base=10000.0), dict(dims=6, base=500.0, scaling=dict(factor=4.0, original=64, fast=8.0, slow=1.0)),
             dict(dims=64, base=20000.0, scaling=dict(factor=16.0, original=4096, fast=32.0, slow=1.0)),
             dict(dims=8, base=50.0, scaling=dict(factor=1.0, original=128, fast=4.0, slow=2.0)),
             dict(dims=12, base=9.0, scaling=dict(factor=2.0, original=8, fast=300.0, slow=200.0)))   # (lo = hi = 0: a step)


def scaled_frequencies():
    """The ramp at several sizes, with ends outside the pairs and where both ends meet."""
    for rot in ROTATIONS:
        sc = rot.get("scaling")
        for kind in ("partial_rope", "pair_rope"):
            kw = dict(dims=rot["dims"], base=rot["base"], scaling=None if sc is None else dict(sc, kind="ramp"))
            pe = POSITION_ENCODINGS.build(kind, **kw, **({"head_dim": rot["dims"] + 4} if kind == "partial_rope" else {}))
            f, mult = plain.frequencies(rot)
            pe.to_device("cpu")
            got, dims = pe.frequencies()
            assert dims == rot["dims"] and abs(pe.mult - mult) < 1e-12
            assert float((got.double() / f - 1).abs().max()) < 1e-6
    f, mult = plain.frequencies(ROTATIONS[1])
    base = torch.tensor([500.0 ** (-2 * i / 6) for i in range(3)], dtype=torch.float64)
    assert mult > 1.1 and float((f / base - 1).abs().max()) > 0.5     # (the case scales something)


def rotated_inputs(o, device, dtype):
    """Queries and keys behind the projection: the first entries of a head turned, with the factor on sines and cosines,
    the others as they are, at positions that do not start at zero; widths with and without pieces of eight."""
    for rot, dk, dv in ((ROTATIONS[1], 10, 14), (ROTATIONS[0], 16, 8), (ROTATIONS[2], 96, 112), (ROTATIONS[3], 8, 3)):
        H, K, P = 4, 2, 4
        f, mult = plain.frequencies(rot)
        m, T = _meta([5, 1], [0, 1], [37, 900])
        pos = torch.tensor([37, 38, 39, 40, 41, 900])
        proj = rand((T, (H + K) * dk + K * dv + 2), 1).to(dtype)
        k_pages = torch.zeros((20, K, P, dk), dtype=dtype, device=device)
        v_pages = torch.zeros((20, K, dv, P), dtype=dtype, device=device)
        slots = torch.tensor([3 * P + i for i in range(4)] + [7 * P, 9 * P + 2], dtype=torch.int64)
        got = o.attention_inputs(proj.to(device), m.to(device), 2, 5, H, K, dk, dv, inv_freq=f.float().to(device),
                                 rot_dims=rot["dims"], rot_mult=mult, slot_mapping=slots.to(device), k_pages=k_pages, v_pages=v_pages)
        tol = 3e-4 if dtype == torch.float32 else 2e-2     # (32-bit angles of up to 900)
        close(got, plain.rotate_half(proj[:, :H * dk].double().view(T, H, dk), pos, rot).reshape(T, -1), tol, (dk, dv))
        from torch_ops import stored_keys_as_rows

        keys = stored_keys_as_rows(k_pages.cpu())
        want = plain.rotate_half(proj[:, H * dk:(H + K) * dk].double().view(T, K, dk), pos, rot)
        for t in range(T):
            page, off = int(slots[t]) // P, int(slots[t]) % P
            close(keys[page, :, off], want[t], tol, ("key", dk, t))
            close(v_pages[page, :, :, off], proj[t, (H + K) * dk:(H + K) * dk + K * dv].view(K, dv), 0.0, ("value", dk, t))


def _attention_part(device, dtype, sizes, std, window, rot, scale=0.3, alter=None):
    D, H, K, dk, dv = sizes
    m = {"heads": H, "kv_heads": K, "dim": dk, "vdim": dv, "scale": scale}
    if window:
        m["mask"] = {"size": window}
    pe = None
    if rot:
        m["rot"] = rot
        sc = rot.get("scaling")
        pe = PartSpec("partial_rope", {"head_dim": dk, "dims": rot["dims"], "base": rot["base"],
                                       "scaling": None if sc is None else dict(sc, kind="ramp")})
    p = {"q": rand((H * dk, D), 50, std), "k": rand((K * dk, D), 51, std), "v": rand((K * dv, D), 52, std), "o": rand((D, H * dv), 53, std)}
    if alter is not None:
        alter(p)
    part = MIXERS.build("gated_attention", hidden_size=D, num_heads=H, num_kv_heads=K, key_dim=dk, value_dim=dv, scale=scale,
                        output_gate=None, window=window, position_encoding=pe)
    _load(part, {n + "_proj": p[n] for n in "qkvo"}, dtype, device)
    return part, {"p." + n: t.to(dtype).double() for n, t in p.items()}, m


def attention_part(device, dtype, sizes=(40, 6, 2, 10, 14), window=9, rot=ROTATIONS[1], page_size=4, length=61, cuts=CUTS, std=0.3):
    part, w, m = _attention_part(device, dtype, sizes, std, window, rot)
    x = rand((length, sizes[0]), 57).to(dtype)
    want = plain.attention(w, "p.", m, x.double(), 1e-5)
    for c in cuts:
        got = run_mixer(part, x.to(device), c, dtype, device, page_size)
        close(got, want, 2e-5 if dtype == torch.float32 else 5e-2, (sizes, window, c[:4]))


def window_edges(device, dtype, sizes=(40, 6, 2, 10, 14), window=37, page_size=16, T=120, std=0.3):
    """One key made to stand out for the last token's query, through entries that are not rotated: just inside the window
    (it decides the result), just outside (it must not be seen), one further, the token itself, page borders, far back
    where there is no window; the query in a prompt's portion and decoded alone."""
    D, H, K, dk, dv = sizes

    def alter(p):
        # input channel 0 makes the queries' last entry, channel 1 the keys'
        p["q"][:, :2] = 0.0
        p["k"][:, :2] = 0.0
        for h in range(H):
            p["q"][h * dk + dk - 1] = 0.0
            p["q"][h * dk + dk - 1, 0] = 5.0
        for h in range(K):
            p["k"][h * dk + dk - 1] = 0.0
            p["k"][h * dk + dk - 1, 1] = 5.0

    rot = dict(dims=dk // 2 // 2 * 2, base=10000.0)
    backs = (window - 2, window - 1, window, window + 1, 0) if window else (T - 1, T - 2, 60, 17, 1)
    for back in backs:
        part, w, m = _attention_part(device, dtype, sizes, std, window, rot, alter=alter)
        key = T - 1 - back
        x = rand((T, D), 58, 0.5)
        x[:, :2] = 0.0
        x[T - 1, 0] = 6.0
        x[key, 1] = 6.0
        x = x.to(dtype)
        want = plain.attention(w, "p.", m, x.double(), 1e-5)
        # the comparison is sharp: a window one off gives another result where the key stands at its edge
        if window and back in (window - 1, window):
            other = plain.attention(w, "p.", dict(m, mask={"size": window + (1 if back == window else -1)}), x.double(), 1e-5)
            assert float((other - want)[-1].abs().max() / want[-1].abs().max()) > 0.3
        for c in ([T], [T - 1, 1], [T // 3, T // 3, T - 2 * (T // 3) - 2, 2]):
            close(run_mixer(part, x.to(device), c, dtype, device, page_size)[-1:], want[-1:],
                  3e-5 if dtype == torch.float32 else 5e-2, (window, back, c))


# --------------------------------------------------------------------------- router, feed-forwards
def router_among_the_chosen(o, device, dtype=torch.float32):
    """Logits with a bias, the softmax over the chosen ones alone: made cases (a bias that turns the choice around, logits so
    far apart that a softmax over all experts would round the smaller ones to zero) and drawn ones."""
    far = torch.linspace(400.0, -400.0, 12, dtype=torch.float64).expand(2, 12).clone()
    turned = torch.zeros(12, dtype=torch.float64)
    turned[7], turned[3] = 900.0, 890.0
    cases = [(far, torch.zeros(12, dtype=torch.float64), 3), (far, turned, 2)]
    for seed, (E, top) in enumerate([(8, 2), (6, 6), (1, 1), (5, 3), (64, 6), (130, 3), (512, 70)]):
        cases.append((rand((33, E), 10 + seed, 2.0), rand((E,), 30 + seed, 3.0), top))
    for z, bias, top in cases:
        z, bias = z.float(), bias.to(torch.bfloat16)
        e, w = o.route_choice(z.to(device), top, 1.0, softmax="chosen", bias=bias.to(device))
        e, w = e.cpu().tolist(), w.cpu().double()
        for t in range(z.shape[0]):
            want = dict(plain.choose((z[t] + bias.float()).double(), top))
            assert sorted(e[t]) == sorted(want), (t, top)
            for i, expert in enumerate(e[t]):
                assert abs(float(w[t, i]) - float(want[expert])) < 2e-6, (t, expert)
    e, _ = o.route_choice(far[:1].float().to(device), 2, 1.0, softmax="chosen", bias=turned.float().to(device))
    assert e.cpu()[0].tolist() == [3, 7]


def routed_part(device, dtype, experts=6, top=3, ff=24, width=40, T=70):
    D = width
    w = {"p.router": rand((experts, D), 1), "p.router.b": rand((experts,), 2, 2.0)}
    for e in range(experts):
        w |= {f"p.e{e}.gate": rand((ff, D), 100 + e, 0.3), f"p.e{e}.up": rand((ff, D), 200 + e, 0.3),
              f"p.e{e}.down": rand((D, ff), 300 + e, 0.3)}
    names = {"router": "p.router", "router_bias": "p.router.b"} | \
        {f"e{e}.{n}": f"p.e{e}.{n}" for e in range(experts) for n in ("gate", "up", "down")}
    part = FEED_FORWARDS.build("routed_experts", hidden_size=D, num_experts=experts, top=top, expert_size=ff, router="chosen_softmax",
                               router_bias=True, activation="silu")
    _load(part, {local: w[name] for local, name in names.items()}, dtype, device)
    x = rand((T, D), 5).to(dtype)
    mlp = {"expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    want = plain.moe({k: v.to(dtype).double() for k, v in w.items()}, "p.", mlp, x.double())
    got = part.forward(x.to(device), None)
    rows = (got.double().cpu() - want).abs().amax(-1) / want.abs().max()
    # (a bfloat16 run may take another expert where two logits are close: a few rows at most)
    tol = 2e-5 if dtype == torch.float32 else 5e-2
    assert int((rows > tol).sum()) <= (0 if dtype == torch.float32 else 3), float(rows.max())
    alone = torch.cat([part.forward(x[t:t + 1].to(device), None) for t in (0, 1, T - 1)])   # (a row does not feel its batch)
    close(alone, got.cpu()[[0, 1, T - 1]], tol, "rows alone")


def dense_part(device, dtype):
    for T, D, F in ((5, 40, 28), (70, 64, 96), (1, 30, 20)):
        w = {"p.up": rand((F, D), 1, 0.3), "p.down": rand((D, F), 2, 0.3)}
        part = FEED_FORWARDS.build("dense", hidden_size=D, intermediate_size=F, activation="squared_relu")
        _load(part, {"up_proj": w["p.up"], "down_proj": w["p.down"]}, dtype, device)
        x = rand((T, D), 3).to(dtype)
        want = plain.dense({k: v.to(dtype).double() for k, v in w.items()}, "p.", x.double())
        close(part.forward(x.to(device), None), want, 2e-5 if dtype == torch.float32 else 3e-2, (T, D, F))


def parts_refuse_what_does_not_fit():
    import pytest

    for kind, registry, kw in (
            ("state_space", MIXERS, dict(hidden_size=8, num_heads=3, num_groups=2, state_dim=4, value_dim=4, conv_taps=4, norm_groups=1, norm_eps=1e-5)),
            ("state_space", MIXERS, dict(hidden_size=8, num_heads=2, num_groups=2, state_dim=4, value_dim=4, conv_taps=0, norm_groups=1, norm_eps=1e-5)),
            ("state_space", MIXERS, dict(hidden_size=8, num_heads=2, num_groups=2, state_dim=4, value_dim=4, conv_taps=4, norm_groups=3, norm_eps=1e-5)),
            ("routed_experts", FEED_FORWARDS, dict(hidden_size=8, num_experts=4, top=2, expert_size=8, router="chosen_softmax", renormalize=1e-9)),
            ("routed_experts", FEED_FORWARDS, dict(hidden_size=8, num_experts=4, top=2, expert_size=8, router="largest")),
            ("partial_rope", POSITION_ENCODINGS, dict(head_dim=8, dims=8, base=10.0, scaling={"kind": "curve"})),
            ("partial_rope", POSITION_ENCODINGS, dict(head_dim=8, dims=8, base=10.0, scaling={"kind": "ramp", "factor": 2.0})),
            ("sink_attention", MIXERS, dict(hidden_size=8, num_heads=2, num_kv_heads=1, key_dim=8, value_dim=8, scale=1.0,
                                            position_encoding=PartSpec("partial_rope", {"head_dim": 8, "dims": 8, "base": 10.0, "scaling": {
                                                "kind": "ramp", "factor": 2.0, "original": 64, "fast": 8.0, "slow": 1.0}})))):
        with pytest.raises(ValueError):
            registry.build(kind, **kw)
