"""A plain, slow implementation of Kolorax, written from the design's equations: one function per mechanism, whole
sequences at a time, recurrences token by token, everything in the element type that it is called with (float64 in the
tests).  It shares no code with the package.

`w` maps tensor names to tensors, `cfg` is the dictionary of config.json.
"""
from __future__ import annotations

import torch


def rms_unit(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x, weight, bias, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * weight + bias


def norm(w, name, x, eps):
    return layer_norm(x, w[name], w[name + ".b"], eps)


def silu(z):
    return z * torch.sigmoid(z)


# ---------------------------------------------------------------------------------------------- loop
def schedule(cfg):
    """[(layer, pass that begins in front of it or None)]"""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    order = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        order += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return order + [(i, None) for i in range(loop["stop"], n)]


def begin_pass(w, t, x, x0):
    return torch.cat([x, x0], -1) @ w["loop.in"].T + w["loop.step"][t]


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


# ---------------------------------------------------------------------------------------------- latent attention
def rotate_half(x, positions, dims, base):
    """x [T, ..., n]: the first `dims` entries of the last axis turn in pairs (i, i + dims / 2)."""
    half = dims // 2
    f = base ** (-2.0 * torch.arange(half, dtype=torch.float64) / dims)
    ang = positions.to(torch.float64)[:, None] * f
    ang = ang.reshape(ang.shape[0], *([1] * (x.dim() - 2)), half)
    c, s = torch.cos(ang).to(x.dtype), torch.sin(ang).to(x.dtype)
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., dims:]], -1)


def latent_attention(w, p, m, h, eps):
    T, H, dk, dr, dv, R = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos = torch.arange(T)
    q = (h @ w[p + "q"].T).view(T, H, dk + dr)
    down = h @ w[p + "dkv"].T
    c = rms_unit(down[:, :R], eps) * w[p + "dkv.norm"]
    kr = down[:, R:]
    qu, qr = q[..., :dk], q[..., dk:]
    if m.get("rot"):
        dims, base = m["rot"].get("dims", dr), m["rot"]["base"]
        qr, kr = rotate_half(qr, pos, dims, base), rotate_half(kr, pos, dims, base)
    ku = (c @ w[p + "uk"].T).view(T, H, dk)
    v = (c @ w[p + "uv"].T).view(T, H, dv)
    seen = pos[None, :] <= pos[:, None]
    out = []
    for a in range(H):
        s = (qu[:, a] @ ku[:, a].T + qr[:, a] @ kr.T) * m["scale"]
        out.append(torch.softmax(s.masked_fill(~seen, float("-inf")), -1) @ v[:, a])
    o = torch.cat(out, -1) * torch.sigmoid(h @ w[p + "g"].T)
    return o @ w[p + "o"].T


# ---------------------------------------------------------------------------------------------- feed-forward
def clamped_glu(gate, up, limit):
    g, u = gate.clamp(max=limit), up.clamp(-limit, limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1)


def expert(w, p, h, limit):
    return clamped_glu(h @ w[p + "gate"].T, h @ w[p + "up"].T, limit) @ w[p + "down"].T


def choose(z, router):
    """z [E]: one token's logits.  Returns [(expert, weight)]."""
    s = torch.softmax(z, -1)
    E, groups = s.shape[0], router.get("groups") or {"count": 1, "keep": 1}
    per = E // groups["count"]
    best = sorted(range(groups["count"]), key=lambda g: (-float(s[g * per:(g + 1) * per].max()), g))[:groups["keep"]]
    allowed = [e for e in range(E) if e // per in best]
    chosen = sorted(allowed, key=lambda e: (-float(s[e]), e))[:router["top"]]
    total = sum(s[e] for e in chosen) + 1e-20
    return [(e, s[e] / total) for e in chosen]


def moe(w, p, mlp, h):
    z = h @ w[p + "router"].T
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, weight in choose(z[t], mlp["router"]):
            y[t] += weight * expert(w, f"{p}e{e}.", h[t:t + 1], mlp["expert"]["limit"])[0]
    if mlp.get("shared") is not None:
        y = y + expert(w, p + "shared.", h, mlp["shared"]["limit"])
    return y


# ---------------------------------------------------------------------------------------------- the model
MIXERS = {"wkv": wkv, "latent_attention": latent_attention}


def layer(w, cfg, i, x):
    L, eps, m, p = cfg["layers"][i], cfg["norm"]["eps"], cfg["residual_mult"], f"l{i}."
    x = x + m * MIXERS[L["type"]](w, p + "mix.", L["mixer"], norm(w, p + "norm1", x, eps), eps)
    if L.get("mlp") is not None:
        x = x + m * moe(w, p + "mlp.", L["mlp"], norm(w, p + "norm2", x, eps))
    return x


def forward(w, cfg, tokens, dtype=torch.float64, layers_out: list | None = None):
    """Logits [T, vocab] of a whole sequence.  `layers_out` collects the stream after every layer run."""
    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in w.items()}
    x0 = w["embed"][torch.tensor([int(t) for t in tokens])] * cfg["embedding"]["scale"]
    x = x0
    for i, t in schedule(cfg):
        if t is not None:
            x = begin_pass(w, t, x, x0)
        x = layer(w, cfg, i, x)
        if layers_out is not None:
            layers_out.append(x.clone())
    return norm(w, "final.norm", x, cfg["norm"]["eps"]) @ w["head"].T


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
