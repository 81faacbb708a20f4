"""TEST INFRASTRUCTURE: a plain, slow restatement of the Zumuzen decoder, one function per mechanism, in float64 on the CPU: layers that may run several times with the same weights
(the embedding rows and a step vector join the stream in front of every pass), a real-gated linear recurrent unit behind a short convolution, chunked softmax attention (biased
projections, half-split rotary with or without the ramp over pair indices, values that may be the unrotated keys, an optional learned sink), decayed linear attention with SiLU operands,
time mixing with a token shift, per-channel decays from the data and a bonus for the current token, two ways of joining mixers side by side, dense SiLU-GLU feed-forwards.
Shares no code with the product path (mistral.rs_amd/hybrid.py, csrc/hyb_*.hip).

A model is `(cfg, w)`: `cfg` the parsed config dictionary, `w` a dict name -> float64 torch tensor.  Every mixer takes the rows of ONE sequence [T, ...] and the state the sequence carried
before them (None: a fresh sequence), and returns its output and the new state, so the same functions restate whole prompts and token-by-token decoding.
"""
from __future__ import annotations

import math

import torch

F = torch.float64


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def silu(x):
    return x * torch.sigmoid(x)


def gelu_tanh(x):
    return 0.5 * x * (1 + torch.tanh(math.sqrt(2 / math.pi) * (x + 0.044715 * x ** 3)))


def softplus(x):
    return torch.clamp(x, min=0) + torch.log1p(torch.exp(-x.abs()))


# ------------------------------------------------------------------------------------------------------------------ chunked attention
def frequencies(rot):
    """(angular frequency of every pair, multiplier of cos and sin)"""
    n, base, sc = int(rot["dims"]), float(rot["base"]), rot.get("scaling")
    f = [base ** (-2.0 * i / n) for i in range(n // 2)]
    if not sc:
        return f, 1.0
    place = lambda turns: n * math.log(sc["original"] / (2 * math.pi * turns)) / (2 * math.log(base))
    lo, hi = max(math.floor(place(sc["fast"])), 0), min(math.ceil(place(sc["slow"])), n - 1)
    ramp = [min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0) for i in range(n // 2)]
    return [fi / sc["factor"] * r + fi * (1 - r) for fi, r in zip(f, ramp)], 0.1 * math.log(sc["factor"]) + 1.0


def rotate_half(x, pos, rot):
    """x [T, H, D]; the pair (i, i + dims / 2) of every head turns by position * frequency"""
    if not rot or not rot["dims"]:
        return x
    f, mult = frequencies(rot)
    h = rot["dims"] // 2
    ang = pos.to(F)[:, None] * torch.tensor(f, dtype=F)
    c, s = torch.cos(ang)[:, None, :] * mult, torch.sin(ang)[:, None, :] * mult
    u, v = x[..., :h], x[..., h:2 * h]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * h:]], -1)


def attend(q, k, v, p0, scale, chunk, sink=None):
    """q [T, H, D] at positions p0 ..; k [N, G, D], v [N, G, Dv] of all positions 0 .. N - 1.  A query sees the keys of its own chunk up to itself; sink [H]: a further term
    e^sink in the denominator."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=F)
    for t in range(T):
        i = p0 + t
        lo = (i // chunk) * chunk if chunk else 0
        for h in range(H):
            g = h // (H // G)
            s = (k[lo:i + 1, g] @ q[t, h]) * scale
            top = s.max() if sink is None else torch.maximum(s.max(), sink[h])
            e = torch.exp(s - top)
            den = e.sum() + (torch.exp(sink[h] - top) if sink is not None else 0.0)
            out[t, h] = (e / den) @ v[lo:i + 1, g]
    return out


def attention(h, w, p, m, st, p0, values_are_keys=False, sink=False):
    """st: (keys, values) of the positions before p0"""
    T, H, G, D = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    Dv = D if values_are_keys else m["vdim"]
    q = (h @ w[p + "q"].T + w[p + "q.b"]).view(T, H, D)
    k = (h @ w[p + "k"].T + w[p + "k.b"]).view(T, G, D)
    v = k if values_are_keys else (h @ w[p + "v"].T + w[p + "v.b"]).view(T, G, Dv)
    pos = torch.arange(p0, p0 + T)
    q, k = rotate_half(q, pos, m.get("rot")), rotate_half(k, pos, m.get("rot"))
    if st is not None:
        k, v = torch.cat([st[0], k]), torch.cat([st[1], v])
    o = attend(q, k, v, p0, float(m["scale"]), int((m.get("mask") or {}).get("size", 0)), w[p + "sink"] if sink else None)
    return o.reshape(T, H * Dv) @ w[p + "o"].T, (k, v)


# ------------------------------------------------------------------------------------------------------------------ decayed linear attention
def decayed_cell(q, k, v, decay, S):
    """q, k [T, H, D]; v [T, H, Dv]; decay [H]; S [H, D, Dv].  Per row: S <- decay_h S + k v^T; o = S^T q."""
    S, out = S.clone(), torch.zeros(q.shape[0], q.shape[1], v.shape[2], dtype=F)
    for t in range(q.shape[0]):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (q[t][:, None, :] @ S)[:, 0]
    return out, S


def lightning(h, w, p, m, eps, S):
    T, H, D, Dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q, k, v = silu(h @ w[p + "q"].T).view(T, H, D), silu(h @ w[p + "k"].T).view(T, H, D), silu(h @ w[p + "v"].T).view(T, H, Dv)
    o, S = decayed_cell(q, k, v, torch.tensor(m["decay"], dtype=F), S if S is not None else torch.zeros(H, D, Dv, dtype=F))
    o = rms_norm(o.reshape(T, H * Dv), w[p + "norm"], eps) * torch.sigmoid(h @ w[p + "g"].T)
    return o @ w[p + "o"].T, S


# ------------------------------------------------------------------------------------------------------------------ time mixing
def shifted(h, last):
    """every row's predecessor: the carried row (zeros for a fresh sequence) in front of the rows"""
    first = torch.zeros_like(h[:1]) if last is None else last[None]
    return torch.cat([first, h[:-1]])


def bonus_cell(r, k, v, dec, u, S):
    """r, k, dec [T, H, D]; v [T, H, Dv]; u [H, D]; S [H, D, Dv].  o = (S + diag(u) k v^T)^T r; then S <- diag(dec) S + k v^T."""
    S, out = S.clone(), torch.zeros(r.shape[0], r.shape[1], v.shape[2], dtype=F)
    for t in range(r.shape[0]):
        kv = k[t][:, :, None] * v[t][:, None, :]
        out[t] = (r[t][:, None, :] @ (S + u[:, :, None] * kv))[:, 0]
        S = dec[t][:, :, None] * S + kv
    return out, S


def time_mix(h, w, p, m, eps, st):
    """st: (the last row before, S)"""
    T, H, D = h.shape[0], m["heads"], m["dim"]
    prev = shifted(h, st[0] if st is not None else None)
    mix = lambda n: h + (prev - h) * w[p + "mu." + n]
    r, k, v = ((mix(n) @ w[p + n].T).view(T, H, D) for n in ("r", "k", "v"))
    gate = silu(mix("g") @ w[p + "g"].T)
    z = torch.tanh(mix("w") @ w[p + "w1"].T) @ w[p + "w2"].T + w[p + "w0"]
    o, S = bonus_cell(r, k, v, torch.exp(-torch.exp(z)).view(T, H, D), w[p + "u"], st[1] if st is not None else torch.zeros(H, D, D, dtype=F))
    o = rms_norm(o, 1.0, eps).reshape(T, H * D) * w[p + "norm"] * gate
    return o @ w[p + "o"].T, (h[-1], S)


# ------------------------------------------------------------------------------------------------------------------ recurrent block
def causal_conv(x, cw, cb, past):
    """x [T, C]; cw [C, taps], last column = the current row; past [taps - 1, C]"""
    taps, full = cw.shape[1], torch.cat([past, x])
    out = torch.stack([sum(cw[:, j] * full[t + j] for j in range(taps)) + cb for t in range(x.shape[0])])
    return out, full[full.shape[0] - (taps - 1):]


def rglru_cell(u, r, i, lam, S):
    """u, r, i [T, C]; S [C].  a = exp(-8 r softplus(lam)); S <- a S + sqrt(1 - a^2) i u; all states are returned."""
    out = torch.zeros_like(u)
    for t in range(u.shape[0]):
        log_a = -8.0 * r[t] * softplus(lam)
        S = torch.exp(log_a) * S + torch.sqrt(-torch.expm1(2 * log_a)) * i[t] * u[t]
        out[t] = S
    return out, S


def block_gate(u, wm, b):
    """u [T, C] in equal parts, part j through the square matrix wm[j] plus b[j], sigmoid"""
    n, s, _ = wm.shape
    return torch.sigmoid(torch.cat([u[:, j * s:(j + 1) * s] @ wm[j].T + b[j] for j in range(n)], -1))


def rglru(h, w, p, m, st):
    """st: (the convolution's last inputs, S)"""
    C, taps = m["width"], m["conv"]
    past, S = st if st is not None else (torch.zeros(taps - 1, C, dtype=F), torch.zeros(C, dtype=F))
    y = gelu_tanh(h @ w[p + "y"].T + w[p + "y.b"])
    u, past = causal_conv(h @ w[p + "x"].T + w[p + "x.b"], w[p + "conv"], w[p + "conv.b"], past)
    s, S = rglru_cell(u, block_gate(u, w[p + "ra"], w[p + "ra.b"]), block_gate(u, w[p + "ri"], w[p + "ri.b"]), w[p + "lam"], S)
    return (s * y) @ w[p + "o"].T, (past, S)


# ------------------------------------------------------------------------------------------------------------------ layers, passes, model
def mixer(h, L, w, p, eps, st, p0):
    m, kind = L["mixer"], L["type"]
    if kind == "rglru":
        return rglru(h, w, p, m, st)
    a, b = st if st is not None else (None, None)
    if kind == "parallel":
        l, a = attention(h, w, p + "left.", m["left"], a, p0)
        r, b = lightning(h, w, p + "right.", m["right"], eps, b)
        return (rms_norm(l, w[p + "left.out"], eps) + rms_norm(r, w[p + "right.out"], eps)) / 2, (a, b)
    l, a = attention(h, w, p + "left.", m["left"], a, p0, values_are_keys=True, sink=True)
    r, b = time_mix(h, w, p + "right.", m["right"], eps, b)
    return float(m["left_scale"]) * l + float(m["right_scale"]) * r, (a, b)


def feed_forward(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def passes(cfg):
    """the layers in the order they run: (layer index, pass number in front of which the stream is joined | None)"""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, None) for i in range(n)]
    a, b = lp["start"], lp["stop"]
    return [(i, None) for i in range(a)] + [(i, t if i == a else None) for t in range(lp["times"]) for i in range(a, b)] + [(i, None) for i in range(b, n)]


def forward(cfg, w, tokens, state=None, pos0=0):
    """logits [T, vocab], the stream after every layer run [runs, T, width], the state after the last token"""
    eps = float(cfg["norm"]["eps"])
    emb = w["embed"][torch.as_tensor(tokens)]
    x, after, new = emb, [], []
    for j, (i, t) in enumerate(passes(cfg)):
        L, p = cfg["layers"][i], f"l{i}."
        if t is not None:
            x = x + (emb if t else 0.0) + w["loop.step"][t]
        o, st = mixer(rms_norm(x, w[p + "norm1"], eps), L, w, p + "mix.", eps, state[j] if state is not None else None, pos0)
        new.append(st)
        x = x + o
        if L.get("mlp"):
            x = x + feed_forward(rms_norm(x, w[p + "norm2"], eps), w, p + "mlp.")
        after.append(x)
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T, torch.stack(after), new
