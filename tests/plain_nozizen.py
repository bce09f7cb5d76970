"""A plain, slow implementation of Nozizen, written from the design's equations: one function per mechanism, whole
sequences at a time, recurrences token by token, everything in the element type that it is called with (float64 in the
tests).  It shares no code with the package.

`w` maps tensor names to tensors, `cfg` is the dictionary of config.json.
"""
from __future__ import annotations

import math

import torch


def rms_unit(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x, weight, eps):
    return rms_unit(x, eps) * weight


def silu(z):
    return z * torch.sigmoid(z)


# ---------------------------------------------------------------------------------------------- order of layers, streams
def schedule(cfg):
    """The layers in the order in which they run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n))
    again = list(range(loop["start"], loop["stop"])) * loop["times"]
    return list(range(loop["start"])) + again + list(range(loop["stop"], n))


def read_streams(streams, weights):
    """streams [T, s, D] -> the sublayer's input [T, D]."""
    return sum(weights[s] * streams[:, s] for s in range(streams.shape[1]))


def write_streams(streams, mix, out, y):
    """Every stream anew from all of the old ones (mix is [from, to]) and the sublayer's result y [T, D]."""
    n = streams.shape[1]
    return torch.stack([sum(mix[s, t] * streams[:, s] for s in range(n)) + out[t] * y for t in range(n)], 1)


# ---------------------------------------------------------------------------------------------- wkv
def previous(h, first=None):
    """Every row's predecessor; the first row's is `first` (zeros at a sequence's start)."""
    head = torch.zeros_like(h[:1]) if first is None else first[None]
    return torch.cat([head, h[:-1]])


def shifted_mix(h, before, mu):
    return h + (before - h) * mu


def decay(mix, w1, w2, w0):
    return torch.exp(-torch.exp(torch.tanh(mix @ w1.T) @ w2.T + w0))


def wkv_recurrence(r, k, v, a, u, S=None):
    """r, k, a [T, d], v [T, e], u [d]; returns (o [T, e], the state behind the last token)."""
    S = torch.zeros(r.shape[1], v.shape[1], dtype=r.dtype) if S is None else S.clone()
    out = []
    for t in range(r.shape[0]):
        kv = torch.outer(k[t], v[t])
        out.append((S + u[:, None] * kv).T @ r[t])
        S = a[t][:, None] * S + kv
    return torch.stack(out), S


def wkv(w, p, m, h, eps):
    T, H, d = h.shape[0], m["heads"], m["dim"]
    before = previous(h)
    mix = {s: shifted_mix(h, before, w[p + "mu." + s]) for s in "rkvgw"}
    r, k, v = ((mix[s] @ w[p + s].T).view(T, H, d) for s in "rkv")
    gate = silu(mix["g"] @ w[p + "g"].T)
    a = decay(mix["w"], w[p + "w1"], w[p + "w2"], w[p + "w0"]).view(T, H, d)
    heads = [wkv_recurrence(r[:, i], k[:, i], v[:, i], a[:, i], w[p + "u"][i])[0] for i in range(H)]
    o = torch.cat([rms_unit(o, eps) for o in heads], -1)
    return (o * w[p + "norm"] * gate) @ w[p + "o"].T


# ---------------------------------------------------------------------------------------------- mamba2
def causal_conv(x, taps, bias, before=None):
    """x [T, C], taps [C, n] with the current token's last; before [n - 1, C] are the inputs in front of the first row."""
    n = taps.shape[1]
    pad = torch.zeros(n - 1, x.shape[1], dtype=x.dtype) if before is None else before
    xs = torch.cat([pad, x])
    return silu(sum(xs[j:j + x.shape[0]] * taps[:, j] for j in range(n)) + bias)


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def ssd_recurrence(x, B, C, dt, a_log, d, S=None):
    """One head: x [T, v], B, C [T, N], dt [T], a_log and d numbers; returns (y [T, v], the state behind the last token)."""
    S = torch.zeros(B.shape[1], x.shape[1], dtype=x.dtype) if S is None else S.clone()
    out = []
    for t in range(x.shape[0]):
        S = torch.exp(-torch.exp(a_log) * dt[t]) * S + dt[t] * torch.outer(B[t], x[t])
        out.append(S.T @ C[t] + d * x[t])
    return torch.stack(out), S


def gated_group_norm(y, z, groups, weight, eps):
    """The gate first, then every group of channels by its own root mean square."""
    g = (y * silu(z)).reshape(y.shape[0], groups, -1)
    return rms_unit(g, eps).reshape(y.shape) * weight


def mamba2(w, p, m, h, eps):
    T, H, N, G, dv = h.shape[0], m["heads"], m["state"], m["groups"], m["vdim"]
    inner = H * dv
    z, xbc, dt = torch.split(h @ w[p + "in"].T, [inner, inner + 2 * G * N, H], -1)
    xbc = causal_conv(xbc, w[p + "conv"], w[p + "conv.b"])
    x, B, C = torch.split(xbc, [inner, G * N, G * N], -1)
    x, B, C = x.reshape(T, H, dv), B.reshape(T, G, N), C.reshape(T, G, N)
    dt = softplus(dt + w[p + "dt_bias"])
    heads = []
    for i in range(H):
        g = i // (H // G)
        heads.append(ssd_recurrence(x[:, i], B[:, g], C[:, g], dt[:, i], w[p + "A_log"][i], w[p + "D"][i])[0])
    return gated_group_norm(torch.cat(heads, -1), z, m["norm_groups"], w[p + "norm"], eps) @ w[p + "o"].T


# ---------------------------------------------------------------------------------------------- attention
def frequencies(rot):
    """(one frequency per pair, the factor on cosines and sines)."""
    dims, base = rot["dims"], rot["base"]
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return torch.tensor(f, dtype=torch.float64), 1.0

    def at(turns):
        return dims * math.log(sc["original"] / (2 * math.pi * turns)) / (2 * math.log(base))

    lo, hi = max(math.floor(at(sc["fast"])), 0), min(math.ceil(at(sc["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * ramp + fi * (1 - ramp))
    return torch.tensor(out, dtype=torch.float64), 0.1 * math.log(sc["factor"]) + 1.0


def rotate_half(x, positions, rot):
    """x [T, ..., n]: the first `dims` entries of the last axis turn in pairs (i, i + dims / 2)."""
    half, dims = rot["dims"] // 2, rot["dims"]
    f, mult = frequencies(rot)
    ang = positions.to(torch.float64)[:, None] * f
    ang = ang.reshape(ang.shape[0], *([1] * (x.dim() - 2)), half)
    c, s = (mult * torch.cos(ang)).to(x.dtype), (mult * torch.sin(ang)).to(x.dtype)
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., dims:]], -1)


def visible(T, window):
    """[T, T]: whether position i (row) sees position j."""
    back = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    return (back >= 0) & (back < window) if window else back >= 0


def attention(w, p, m, h, eps):
    T, H, G, dk, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos = torch.arange(T)
    q, k, v = ((h @ w[p + n].T).view(T, a, b) for n, a, b in (("q", H, dk), ("k", G, dk), ("v", G, dv)))
    if m.get("rot"):
        q, k = rotate_half(q, pos, m["rot"]), rotate_half(k, pos, m["rot"])
    seen = visible(T, (m.get("mask") or {}).get("size"))
    out = []
    for a in range(H):
        g = a // (H // G)
        s = (q[:, a] @ k[:, g].T) * m["scale"]
        out.append(torch.softmax(s.masked_fill(~seen, float("-inf")), -1) @ v[:, g])
    return torch.cat(out, -1) @ w[p + "o"].T


# ---------------------------------------------------------------------------------------------- feed-forward
def dense(w, p, h):
    return torch.relu(h @ w[p + "up"].T) ** 2 @ w[p + "down"].T


def expert(w, p, h):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def choose(z, top):
    """z [E]: one token's logits.  Returns [(expert, weight)]: the largest logits, and the softmax over these alone."""
    chosen = sorted(range(z.shape[0]), key=lambda e: (-float(z[e]), e))[:top]
    weights = torch.softmax(torch.stack([z[e] for e in chosen]), -1)
    return list(zip(chosen, weights))


def moe(w, p, mlp, h):
    z = h @ w[p + "router"].T + w[p + "router.b"]
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, weight in choose(z[t], mlp["router"]["top"]):
            y[t] += weight * expert(w, f"{p}e{e}.", h[t:t + 1])[0]
    return y


# ---------------------------------------------------------------------------------------------- the model
MIXERS = {"wkv": wkv, "mamba2": mamba2, "attention": attention}


def feed_forward(w, p, mlp, h):
    return dense(w, p, h) if mlp["kind"] == "dense" else moe(w, p, mlp, h)


def sublayer(w, p, q, streams, f, eps):
    """q 1: the mixer, 2: the feed-forward; f: what the sublayer computes from its normed input."""
    u = read_streams(streams, w[f"{p}hc{q}.in"])
    y = f(rms_norm(u, w[f"{p}norm{q}"], eps))
    return write_streams(streams, w[f"{p}hc{q}.mix"], w[f"{p}hc{q}.out"], y)


def layer(w, cfg, i, streams):
    L, eps, p = cfg["layers"][i], cfg["norm"]["eps"], f"l{i}."
    streams = sublayer(w, p, 1, streams, lambda h: MIXERS[L["type"]](w, p + "mix.", L["mixer"], h, eps), eps)
    if L.get("mlp") is not None:
        streams = sublayer(w, p, 2, streams, lambda h: feed_forward(w, p + "mlp.", L["mlp"], h), eps)
    return streams


def forward(w, cfg, tokens, dtype=torch.float64, layers_out: list | None = None):
    """Logits [T, vocab] of a whole sequence.  `layers_out` collects the streams' sum after every layer run."""
    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in w.items()}
    x = w["embed"][torch.tensor([int(t) for t in tokens])] * cfg["embedding"]["scale"]
    streams = torch.stack([x] * cfg["streams"], 1)
    for i in schedule(cfg):
        streams = layer(w, cfg, i, streams)
        if layers_out is not None:
            layers_out.append(streams.sum(1))
    return rms_norm(streams.sum(1), w["final.norm"], cfg["norm"]["eps"]) @ w["embed"].T


def greedy(w, cfg, prompt, steps, dtype=torch.float64):
    tokens = list(prompt)
    for _ in range(steps):
        tokens.append(int(forward(w, cfg, tokens, dtype)[-1].argmax()))
    return tokens[len(prompt):]


def load(model_dir: str):
    """(weights by tensor name as stored, config.json as a dict)."""
    import json
    import os

    from safetensors import safe_open

    with open(os.path.join(model_dir, "config.json")) as f:
        cfg = json.load(f)
    w = {}
    with safe_open(os.path.join(model_dir, "model.safetensors"), framework="pt", device="cpu") as h:
        for name in h.keys():
            w[name] = h.get_tensor(name)
    return w, cfg
