"""TEST INFRASTRUCTURE: a plain, slow restatement of the Kebisun decoder, one function per mechanism, in float64 on the CPU: a scaled embedding, layers whose sublayers read
the residual row as it is and join it through a layer norm (weight, no bias) and a per-channel scale, a gated linear attention mixer (one decay per key channel, an
outer-product state, a per-head output norm, a SiLU gate), a latent attention mixer (query latent, cached latent row beside one rotated key part shared by the heads, YaRN
rotary, sliding window, a learned sink per head, an elementwise sigmoid gate), dense GELU-GLU feed-forwards and routed GELU experts whose weights are the chosen softmax scores.
Shares no code with the product path (mistral.rs_amd/hybrid.py, csrc/hyb_*.hip).

A model is `(cfg, w)`: `cfg` the parsed config dictionary, `w` a dict name -> float64 torch tensor.  Every mixer takes the rows of ONE sequence [T, ...] and the state the
sequence carried before them (None: a fresh sequence), and returns its output and the new state, so the same functions restate whole prompts and token-by-token decoding.
"""
from __future__ import annotations

import math

import torch

F = torch.float64


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def layer_norm(x, w, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w


def silu(x):
    return x * torch.sigmoid(x)


def gelu_tanh(x):
    return 0.5 * x * (1 + torch.tanh(math.sqrt(2 / math.pi) * (x + 0.044715 * x ** 3)))


def gelu_erf(x):
    return 0.5 * x * (1 + torch.erf(x / math.sqrt(2.0)))


# ------------------------------------------------------------------------------------------------------------------ gated linear attention
def gla_cell(q, k, v, alpha, S):
    """q, k, alpha [T, H, D]; v [T, H, Dv]; S [H, D, Dv].  Per row: S <- alpha S (rows of S scaled) + k v^T; o = S^T q."""
    S = S.clone()
    out = torch.zeros(q.shape[0], q.shape[1], v.shape[2], dtype=F)
    for t in range(q.shape[0]):
        S = alpha[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (q[t][:, None, :] @ S)[:, 0]
    return out, S


def gla_decay(h, w, p, m):
    """alpha = sigmoid(A2 (A1 h) + b)^(1 / tau), [T, H, D]"""
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "a2.b"]
    return (torch.sigmoid(z) ** (1.0 / float(m["tau"]))).view(h.shape[0], m["heads"], m["dim"])


def gla_mixer(h, w, p, m, eps, S):
    T, H, D, Dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).view(T, H, D) * D ** -0.5
    k = (h @ w[p + "k"].T).view(T, H, D)
    v = (h @ w[p + "v"].T).view(T, H, Dv)
    o, S = gla_cell(q, k, v, gla_decay(h, w, p, m), S if S is not None else torch.zeros(H, D, Dv, dtype=F))
    o = rms_norm(o, w[p + "norm"], eps).reshape(T, H * Dv) * silu(h @ w[p + "g"].T)
    return o @ w[p + "o"].T, S


# ------------------------------------------------------------------------------------------------------------------ latent attention
def yarn(rot):
    """(frequencies [dims / 2], multiplier of cos and sin)"""
    n, base, sc = int(rot["dims"]), float(rot["base"]), rot.get("scaling")
    f = [base ** (-2.0 * i / n) for i in range(n // 2)]
    if not sc:
        return f, 1.0
    place = lambda turns: n * math.log(sc["original"] / (2 * math.pi * turns)) / (2 * math.log(base))
    lo, hi = max(math.floor(place(sc["fast"])), 0), min(math.ceil(place(sc["slow"])), n - 1)
    out = []
    for i, fi in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * r + fi * (1 - r))
    return out, 0.1 * math.log(sc["factor"]) + 1.0


def rotate_half(x, pos, rot):
    """x [T, ..., R]: in the first dims of the last axis the pair (i, i + dims / 2) turns by pos * f_i"""
    n = int(rot["dims"]) if rot else 0
    if not n:
        return x
    f, mult = yarn(rot)
    ang = pos.to(F)[:, None] * torch.tensor(f, dtype=F)[None, :]
    c, s = torch.cos(ang) * mult, torch.sin(ang) * mult
    while c.dim() < x.dim():
        c, s = c[:, None], s[:, None]
    u, v = x[..., :n // 2], x[..., n // 2:n]
    y = x.clone()
    y[..., :n // 2], y[..., n // 2:n] = u * c - v * s, v * c + u * s
    return y


def softmax_sink(s, sink):
    """s [keys]; the denominator has one more term e^{sink}"""
    top = max(float(s.max()), float(sink))
    e = torch.exp(s - top)
    return e / (e.sum() + math.exp(float(sink) - top))


def latent_mixer(h, w, p, m, eps, state, pos0):
    """state = (latents [P, R], rotated key parts [P, rot_dim]) of the positions before these rows (None: none)."""
    T, H, D, Dr, Dv, R = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos = torch.arange(pos0, pos0 + T)
    q = (rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps) @ w[p + "uq"].T).view(T, H, D + Dr)
    qu, qr = q[..., :D], rotate_half(q[..., D:], pos, m.get("rot"))
    dkv = h @ w[p + "dkv"].T
    c, kr = rms_norm(dkv[:, :R], w[p + "dkv.norm"], eps), rotate_half(dkv[:, R:], pos, m.get("rot"))
    if state is not None:
        c, kr = torch.cat([state[0], c]), torch.cat([state[1], kr])
    ku, v = (c @ w[p + "uk"].T).view(-1, H, D), (c @ w[p + "uv"].T).view(-1, H, Dv)
    size = int((m.get("mask") or {}).get("size", 0) or 0)
    out = torch.zeros(T, H, Dv, dtype=F)
    for t in range(T):
        i = pos0 + t
        lo = max(0, i - size + 1) if size else 0
        for hh in range(H):
            s = (ku[lo:i + 1, hh] @ qu[t, hh] + kr[lo:i + 1] @ qr[t, hh]) * float(m["scale"])
            out[t, hh] = softmax_sink(s, w[p + "sink"][hh]) @ v[lo:i + 1, hh]
    o = out.reshape(T, H * Dv) * torch.sigmoid(h @ w[p + "g"].T)
    return o @ w[p + "o"].T, (c, kr)


# ------------------------------------------------------------------------------------------------------------------ feed-forwards
def glu_ff(h, w, p):
    return (gelu_tanh(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(h, w, p, f):
    """The chosen experts of every row and their weights: softmax over all experts, the `top` largest scores (ties: the lower index), not renormalised."""
    s = torch.softmax(h @ w[p + "router"].T, -1)
    order = torch.sort(s, dim=-1, descending=True, stable=True).indices[:, :int(f["router"]["top"])]
    return order, torch.gather(s, 1, order)


def moe_ff(h, w, p, f):
    ids, wts = route(h, w, p, f)
    out = torch.zeros(h.shape[0], w[p + "e0.down"].shape[0], dtype=F)
    for e in range(int(f["router"]["experts"])):
        t, j = torch.nonzero(ids == e, as_tuple=True)
        if t.numel():
            out[t] += wts[t, j][:, None] * (gelu_erf(h[t] @ w[f"{p}e{e}.up"].T) @ w[f"{p}e{e}.down"].T)
    return out


# ------------------------------------------------------------------------------------------------------------------ the model
def mixer(kind, h, w, p, m, eps, state, pos0):
    if kind == "gla":
        return gla_mixer(h, w, p, m, eps, state)
    if kind == "latent_attention":
        return latent_mixer(h, w, p, m, eps, state, pos0)
    raise ValueError(kind)


def join(x, y, norm, scale, eps):
    """x + scale * norm(y): how a sublayer's output enters the residual stream"""
    return x + layer_norm(y, norm, eps) * scale


def forward(cfg, w, tokens, states=None, pos0=0):
    """Rows `tokens` of one sequence that starts them at position pos0 with the per-layer states `states` (None: fresh).  Returns (logits [T, vocab], the residual stream
    after every layer [L, T, W], new states)."""
    eps = float(cfg["norm"]["eps"])
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * float(cfg["embedding"]["scale"])
    states = list(states) if states is not None else [None] * len(cfg["layers"])
    after = []
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        y, states[i] = mixer(L["type"], x, w, p + "mix.", L["mixer"], eps, states[i], pos0)
        x = join(x, y, w[p + "norm1"], w[p + "ls1"], eps)
        f = L.get("mlp")
        if f:
            y = glu_ff(x, w, p + "mlp.") if f["kind"] == "dense" else moe_ff(x, w, p + "mlp.", f)
            x = join(x, y, w[p + "norm2"], w[p + "ls2"], eps)
        after.append(x)
    return layer_norm(x, w["final.norm"], eps) @ w["head"].T, torch.stack(after), states
