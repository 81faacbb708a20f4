"""Zumuzen decoders (mistralrs_amd.hybrid: layers that run several times, RgLruMixer, LightningMixer, TimeMixMixer, WindowAttention with biases / half-split rotary / keys as values,
ParallelMixer with output scales; csrc/hyb_rglru.hip, csrc/hyb_attn_mfma.hip and the forms added to csrc/hyb_linattn.hip / hyb_kernels.hip) against the plain float64 restatement in
tests/zumuzen_oracle.py.

Every test builds its own small configuration with random bf16-representable weights.  The sharp comparisons run in the all-f32 mode (a wrong key, a lost state, a sink left
out is an O(1) error there, rounding is 1e-6); the bf16 mode (whose prompt attention and recurrence gates run on the matrix cores) is held to a rounding-sized bar, its kernels alone
to the rounding of their result.  CPU tests cover what needs no device.
"""
import io
import json
import math
import os

import numpy as np
import pytest
import torch

import mistralrs_amd  # noqa: F401
from mistralrs_amd import _lib
from tests import zumuzen_oracle as O
from tests.test_kebisun import Served, _batch, close, f64, rel, toks

D64 = torch.float64
BOTH = pytest.mark.parametrize("dtype,bar", [("float32", 5e-5), ("bfloat16", 4e-2)])


# ---------------------------------------------------------------------------------------------------------------- configurations and weights
def dense(ff=56):
    return {"kind": "dense", "ff": ff}


def lru(width=48, blocks=3, conv=4, mlp=56):
    return {"type": "rglru", "mixer": {"width": width, "blocks": blocks, "conv": conv}, "mlp": dense(mlp) if mlp else None}


def par(heads=4, kv=2, dim=16, vdim=24, size=20, dims=16, base=500.0, scale=None, l_heads=3, l_dim=16, l_vdim=8, decay=None, mlp=56):
    return {"type": "parallel", "mlp": dense(mlp) if mlp else None, "mixer": {
        "left": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5, "rot": {"dims": dims, "base": base}, "mask": {"size": size}},
        "right": {"heads": l_heads, "dim": l_dim, "vdim": l_vdim, "decay": decay or [1 - 2.0 ** -(2 + h) for h in range(l_heads)]}}}


def par2(heads=4, kv=2, dim=16, size=20, dims=8, base=300.0, scaling=(4.0, 8.0, 1.0, 64), scale=None, t_heads=3, t_dim=16, ls=0.7, rs=1.3, mlp=56):
    rot = {"dims": dims, "base": base}
    if scaling:
        rot["scaling"] = dict(zip(("factor", "fast", "slow", "original"), scaling))
    return {"type": "parallel_2", "mlp": dense(mlp) if mlp else None, "mixer": {
        "left": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": scale or dim ** -0.5, "rot": rot, "mask": {"size": size}},
        "right": {"heads": t_heads, "dim": t_dim}, "left_scale": ls, "right_scale": rs}}


def config(layers, vocab=96, width=40, eps=1e-5, loop=None):
    c = {"architecture": "Zumuzen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


def weights(cfg, seed=0, rank=5, slow=False):
    """slow: decays close to one, so that a state written early is still read hundreds of tokens later"""
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]
    w = {}

    def rnd(*shape, scale=1.0, shift=0.0):
        return (torch.randn(*shape, generator=g) * scale + shift).to(torch.bfloat16)
    a = W ** -0.5
    w["embed"], w["head"], w["final.norm"] = rnd(cfg["vocab"], W), rnd(cfg["vocab"], W, scale=a), rnd(W, scale=0.2, shift=1.0)
    if cfg.get("loop"):
        w["loop.step"] = rnd(cfg["loop"]["times"], W, scale=0.5)

    def attn(q, m, values_are_keys):
        H, G, D = m["heads"], m["kv_heads"], m["dim"]
        Dv = D if values_are_keys else m["vdim"]
        for n, rows in (("q", H * D), ("k", G * D)) + (() if values_are_keys else (("v", G * Dv),)):
            w[q + n], w[q + n + ".b"] = rnd(rows, W, scale=1.5 * a), rnd(rows, scale=0.5)
        w[q + "o"] = rnd(W, H * Dv, scale=(H * Dv) ** -0.5)
        if values_are_keys:
            w[q + "sink"] = rnd(H, shift=0.5)
    for i, L in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", L["mixer"], L.get("mlp")
        for n in ("1", "2") if f else ("1",):
            w[p + "norm" + n] = rnd(W, scale=0.2, shift=1.0)
        q = p + "mix."
        if L["type"] == "rglru":
            C, B = m["width"], m["blocks"]
            w[q + "y"], w[q + "y.b"], w[q + "x"], w[q + "x.b"] = rnd(C, W, scale=2 * a), rnd(C, scale=0.5), rnd(C, W, scale=2 * a), rnd(C, scale=0.5)
            w[q + "conv"], w[q + "conv.b"] = rnd(C, m["conv"], scale=0.5), rnd(C, scale=0.5)
            for n in ("ra", "ri"):
                w[q + n], w[q + n + ".b"] = rnd(B, C // B, C // B, scale=(C // B) ** -0.5), rnd(B, C // B, scale=0.5)
            w[q + "lam"], w[q + "o"] = rnd(C, scale=0.5, shift=-6.0 if slow else -2.0), rnd(W, C, scale=C ** -0.5)
        else:
            attn(q + "left.", m["left"], L["type"] == "parallel_2")
            r, q = m["right"], q + "right."
            if L["type"] == "parallel":
                nk, nv = r["heads"] * r["dim"], r["heads"] * r["vdim"]
                w[q + "q"], w[q + "k"], w[q + "v"], w[q + "g"] = rnd(nk, W, scale=2 * a), rnd(nk, W, scale=2 * a), rnd(nv, W, scale=2 * a), rnd(nv, W, scale=3 * a)
                w[q + "norm"] = rnd(nv, scale=0.2, shift=1.0)
                for s in ("left", "right"):
                    w[f"{p}mix.{s}.out"] = rnd(W, scale=0.3, shift=1.0)
            else:
                nk = nv = r["heads"] * r["dim"]
                for n in ("r", "k", "v", "g"):
                    w[q + n] = rnd(nk, W, scale=2 * a)
                for n in ("r", "k", "v", "g", "w"):
                    w[q + "mu." + n] = rnd(W, scale=0.3, shift=0.5)
                w[q + "w1"], w[q + "w2"], w[q + "w0"] = rnd(rank, W, scale=a), rnd(nk, rank, scale=rank ** -0.5), rnd(nk, scale=0.5, shift=-6.0 if slow else -1.5)
                w[q + "u"], w[q + "norm"] = rnd(r["heads"], r["dim"]), rnd(nk, scale=0.2, shift=1.0)
            w[q + "o"] = rnd(W, nv, scale=nv ** -0.5)
        if f:
            w[p + "mlp.gate"], w[p + "mlp.up"], w[p + "mlp.down"] = rnd(f["ff"], W, scale=2 * a), rnd(f["ff"], W, scale=2 * a), rnd(W, f["ff"], scale=f["ff"] ** -0.5)
    return w


STACK = [par2(mlp=None), lru(), par(), par2(heads=3, kv=1, dim=24, size=9, dims=24, scaling=None, t_heads=2, t_dim=24), lru(width=40, blocks=1, conv=2, mlp=None), par(heads=2, kv=2, dim=32, vdim=8, dims=8, size=70, mlp=None)]
LOOP = (1, 4, 3)


def logits_of(cfg, wd, t):
    return O.forward(cfg, wd, t)[0]


# ---------------------------------------------------------------------------------------------------------------- no device needed
def test_config_reader_takes_every_size_and_constant_from_the_file():
    from mistralrs_amd.hybrid import AttentionSpec, GluSpec, LightningSpec, RgLruSpec, TimeMixSpec, zumuzen_spec
    cfg = config([lru(width=30, blocks=5, conv=3, mlp=77), par(heads=6, kv=3, dim=10, vdim=14, size=17, dims=4, base=77.0, scale=0.3, l_heads=2, l_dim=6, l_vdim=7, decay=[0.5, 0.25]),
                  par2(heads=4, kv=1, dim=12, size=33, dims=6, base=55.0, scaling=(3.0, 9.0, 2.0, 100), scale=0.2, t_heads=5, t_dim=9, ls=0.6, rs=1.7, mlp=None)], vocab=123, width=56, eps=3e-4)
    sp = zumuzen_spec(cfg)
    assert (sp.vocab, sp.width, sp.eps, sp.norm, sp.head, sp.step, sp.streams, sp.join_norms, sp.post_norms, sp.parallel_sublayers) == (123, 56, 3e-4, "rms", "head", None, 0, False, False, False)
    a, b, c = sp.layers
    assert [l.kind for l in sp.layers] == ["rglru", "parallel", "parallel"] and [l.prefix for l in sp.layers] == ["l0.", "l1.", "l2."]
    assert a.mixer == RgLruSpec(30, 5, 3) and isinstance(a.ff, GluSpec) and (a.ff.ff, a.ff.act) == (77, "silu") and c.ff is None
    m = b.mixer.left
    assert isinstance(m, AttentionSpec) and (m.heads, m.kv_heads, m.dim, m.vdim, m.scale, m.chunk, m.window, m.sink, m.bias, m.values_are_keys, m.qk_norm, m.head_gate) == \
        (6, 3, 10, 14, 0.3, 17, 0, False, True, False, False, False)
    assert (m.rotary.dims, m.rotary.base, m.rotary.layout, m.rotary.scaling) == (4, 77.0, "half", None) and b.mixer.right == LightningSpec(2, 6, 7, [0.5, 0.25]) and b.mixer.scales is None
    m = c.mixer.left
    assert (m.heads, m.kv_heads, m.dim, m.vdim, m.scale, m.chunk, m.sink, m.bias, m.values_are_keys) == (4, 1, 12, 12, 0.2, 33, True, True, True)
    assert (m.rotary.dims, m.rotary.base) == (6, 55.0) and m.rotary.trig_mult == pytest.approx(0.1 * math.log(3.0) + 1.0, abs=1e-12)
    assert c.mixer.right == TimeMixSpec(5, 9) and c.mixer.scales == (0.6, 1.7)
    f, mult = O.frequencies(cfg["layers"][2]["mixer"]["left"]["rot"])
    assert np.allclose(m.rotary.frequencies(), f, rtol=1e-6) and m.rotary.trig_mult == pytest.approx(mult)
    two = par(decay=[0.5])
    for bad in ([{"type": "gla", "mixer": {}, "mlp": None}], [dict(lru(), mlp={"kind": "moe"})], [par(dims=5)], [par(heads=3, kv=2)], [two]):
        with pytest.raises(ValueError):
            zumuzen_spec(config(bad))


def test_looped_layers_become_passes_with_shared_tensors():
    from mistralrs_amd.hybrid import zumuzen_spec
    sp = zumuzen_spec(config([lru(), par(), par2(), lru()], loop=(1, 3, 3)))
    assert [(l.prefix, l.weights_of, l.enter) for l in sp.layers] == [("l0.", None, None), ("l1.", None, 0), ("l2.", None, None), ("l1.", 1, 1), ("l2.", 2, None), ("l1.", 1, 2), ("l2.", 2, None),
                                                                     ("l3.", None, None)]
    assert sp.step == "loop.step" and O.passes(config([lru(), par(), par2(), lru()], loop=(1, 3, 3))) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (1, 2), (2, None), (3, None)]
    sp = zumuzen_spec(config([lru(), par()], loop=(0, 2, 1)))   # one pass: its step vector still joins
    assert [(l.weights_of, l.enter) for l in sp.layers] == [(None, 0), (None, None)] and sp.step == "loop.step"
    sp = zumuzen_spec(config([lru(), par()], loop=(1, 2, 2)))   # a loop of one layer at the end
    assert [(l.prefix, l.weights_of, l.enter) for l in sp.layers] == [("l0.", None, None), ("l1.", None, 0), ("l1.", 1, 1)]
    for bad in ((1, 1, 2), (0, 3, 2), (-1, 1, 2), (0, 1, 0)):
        with pytest.raises(ValueError):
            zumuzen_spec(config([lru(), par()], loop=bad))


def test_registry_and_synthetic_weights_know_the_architecture():
    from mistralrs_amd import registry
    from mistralrs_amd.hybrid import MIXERS, SPEC_READERS, synthetic_weights, zumuzen_spec
    assert "Zumuzen" in registry.ARCHITECTURES and "Zumuzen" in SPEC_READERS and {"rglru", "lightning", "time_mix"} <= set(MIXERS)
    cfg = config(STACK, loop=LOOP)
    get = synthetic_weights(zumuzen_spec(cfg), "cpu", 1)
    for name, t in weights(cfg).items():
        if name.endswith((".w1", ".w2")):
            assert get(name).shape[name.endswith("2") ^ 1] == t.shape[name.endswith("2") ^ 1], name   # the inner size is the generator's choice
        else:
            assert tuple(get(name).shape) == tuple(t.shape), name
    for name in ("l0.norm2", "l0.mix.left.v", "l2.mix.left.sink", "l2.mix.left.q.norm", "l0.mix.left.out"):
        with pytest.raises(KeyError):
            get(name)


def test_restatement_pieces():
    """the oracle's own building blocks on hand-computed values"""
    one = lambda *v: torch.tensor(v, dtype=D64)
    # chunks: position 2 of chunks of two sees itself only, position 3 sees 2 and 3; a sink takes weight and gives nothing
    k, v, q = torch.zeros(4, 1, 1, dtype=D64), one(1, 2, 3, 5).view(4, 1, 1), torch.zeros(4, 1, 1, dtype=D64)
    assert O.attend(q, k, v, 0, 1.0, 2).view(4).tolist() == [1, 1.5, 3, 4] and torch.allclose(O.attend(q, k, v, 0, 1.0, 2, one(math.log(2))).view(4), one(1 / 3, 3 / 4, 1, 2))
    assert O.attend(q[:1], k, v, 3, 1.0, 0).item() == pytest.approx(11 / 4)
    # the state before the row, the row through the bonus; then the decay
    o, S = O.bonus_cell(one(1, 1).view(2, 1, 1), one(2, 3).view(2, 1, 1), one(5, 7).view(2, 1, 1), one(0.5, 0.25).view(2, 1, 1), one(10).view(1, 1), torch.zeros(1, 1, 1, dtype=D64))
    assert o.view(2).tolist() == [100.0, 10.0 + 210.0] and S.item() == 10 * 0.25 + 21
    o, S = O.decayed_cell(one(1, 1).view(2, 1, 1), one(2, 3).view(2, 1, 1), one(5, 7).view(2, 1, 1), one(0.5), torch.zeros(1, 1, 1, dtype=D64))
    assert o.view(2).tolist() == [10.0, 26.0]
    # recurrent unit: r = 0 keeps everything and brings nothing
    u = torch.ones(2, 1, dtype=D64)
    s, S = O.rglru_cell(u, one(0, 1).view(2, 1), u, one(0.0), one(3.0))
    a = math.exp(-8 * math.log(2))
    assert s.view(2).tolist() == pytest.approx([3.0, 3 * a + math.sqrt(1 - a * a)])
    x, past = O.causal_conv(one(1, 2, 3).view(3, 1), one(10, 1).view(1, 2), one(0.5), one(7).view(1, 1))
    assert x.view(3).tolist() == [71.5, 12.5, 23.5] and past.item() == 3
    assert O.shifted(one(1, 2).view(2, 1), None).view(2).tolist() == [0, 1] and O.shifted(one(1, 2).view(2, 1), one(9)).view(2).tolist() == [9, 1]
    x = torch.zeros(3, 1, 6, dtype=D64)
    x[:, 0, 1], x[:, 0, 5] = 1.0, 7.0
    r = O.rotate_half(x, torch.arange(3), {"dims": 4, "base": 100.0})[:, 0]
    assert torch.allclose(r[:, 1], torch.cos(torch.arange(3, dtype=D64) * 0.1)) and torch.allclose(r[:, 3], torch.sin(torch.arange(3, dtype=D64) * 0.1)) and r[:, 5].tolist() == [7.0] * 3
    z = torch.linspace(-3, 3, 7, dtype=D64)
    assert torch.allclose(O.gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh")) and torch.allclose(O.softplus(z), torch.nn.functional.softplus(z))


def test_restatement_decodes_token_by_token_like_whole_prompts():
    cfg = config(STACK, loop=LOOP)
    wd = f64(weights(cfg, 3))
    t = toks(60, cfg["vocab"], 4)
    want, after, _ = O.forward(cfg, wd, t)
    got, st, at = [], None, 0
    for n in (1, 2, 20, 1, 36):
        lg, _, st = O.forward(cfg, wd, t[at:at + n], st, at)
        got.append(lg)
        at += n
    assert rel(torch.cat(got), want) < 1e-12 and after.shape == (len(STACK) + 6, 60, cfg["width"])


# ---------------------------------------------------------------------------------------------------------------- kernels alone (GPU)
@pytest.mark.gpu
@pytest.mark.parametrize("W", [40, 257, 1100, 2049, 4100])
def test_pass_entry_and_normed_average_with_the_next_norm(dev, W):
    from mistralrs_amd.hybrid import _call
    _lib.load("hybrid")
    g = torch.Generator().manual_seed(W)
    T, V = 5, 11
    x0, step, w, w1, w2, y1, y2 = (torch.randn(*s, generator=g) for s in ((T, W), (W,), (W,), (W,), (W,), (T, W), (T, W)))
    ids = torch.tensor([3, 10, 0, 3, 7], dtype=torch.int32)
    for dt, TT in ((2, torch.float32), (1, torch.bfloat16)):
        table = torch.randn(V, W, generator=g).to(torch.bfloat16).to(TT)
        for emb in (False, True):
            for one_plus in (0, 1):
                x, out, o32 = x0.to(dev), torch.empty(T, W, dtype=TT, device=dev), torch.empty(T, W, device=dev)
                _call("mrs_hyb_pass_norm", x, ids.to(dev), table.to(dev) if emb else None, V, 1.0, step.to(dev), w.to(dev), out, o32, T, W, 1e-5, one_plus, dt)
                want = x0.double() + (table.double()[ids.long()] if emb else 0) + step.double()
                assert rel(x.double().cpu(), want) < 1e-6 and rel(o32.double().cpu(), O.rms_norm(want, w.double() + one_plus, 1e-5)) < 2e-6 and torch.equal(out.cpu(), o32.cpu().to(TT))
        avg = 0.5 * (O.rms_norm(y1.double(), w1.double(), 1e-5) + O.rms_norm(y2.double(), w2.double(), 1e-5))
        for acc in (0, 1):
            x, out, o32 = x0.to(dev), torch.empty(T, W, dtype=TT, device=dev), torch.empty(T, W, device=dev)
            _call("mrs_hyb_norm_pair_add_norm", x, W, y1.to(dev), w1.to(dev), y2.to(dev), w2.to(dev), T, W, 1e-5, 0.5, acc, w.to(dev), 0, out, o32, dt)
            want = avg + acc * x0.double()
            assert rel(x.double().cpu(), want) < 1e-6 and rel(o32.double().cpu(), O.rms_norm(want, w.double(), 1e-5)) < 2e-6 and torch.equal(out.cpu(), o32.cpu().to(TT))
            x = x0.to(dev)
            _call("mrs_hyb_norm_pair_add", x, W, y1.to(dev), w1.to(dev), y2.to(dev), w2.to(dev), T, W, 1e-5, 0.5, acc)
            assert rel(x.double().cpu(), want) < 1e-6
        # the norm over all heads with a sigmoid gate behind it, and without
        gate = torch.randn(T, W + 3, generator=g)
        for mode in (1, 2):
            out = torch.empty(T, W, device=dev)
            _call("mrs_hyb_rmsnorm", y1.to(dev), W, w.to(dev), None, out, None, T, W, 1, 1e-5, 0, dt, gate.to(dev), W + 3, mode)
            gd = gate.double()[:, :W]
            assert rel(out.double().cpu(), O.rms_norm(y1.double(), w.double(), 1e-5) * (torch.sigmoid(gd) if mode == 2 else O.silu(gd))) < 2e-6


@pytest.mark.gpu
@pytest.mark.parametrize("M", [1, 5, 8, 9, 300])
def test_products_that_join_with_a_factor(dev, M):
    from mistralrs_amd.hybrid import _call
    _lib.load("hybrid")
    g = torch.Generator().manual_seed(M)
    for N, K in ((40, 72), (150, 33), (129, 256)):
        for dt, TT in ((2, torch.float32), (1, torch.bfloat16)):
            a, w, c = torch.randn(M, K, generator=g).to(TT), torch.randn(N, K, generator=g).to(TT), torch.randn(M, N, generator=g)
            for acc in (0, 1):
                out = c.to(dev)
                _call("mrs_hyb_gemm_scaled", a.to(dev), w.to(dev), out, M, N, K, K, K, N, dt, acc, -0.7)
                assert rel(out.double().cpu(), acc * c.double() - 0.7 * (a.double() @ w.double().T)) < 3e-6


@pytest.mark.gpu
@pytest.mark.parametrize("dt", [2, 1], ids=["f32", "bf16"])
@pytest.mark.parametrize("H,G,D,Dv,dims,own_v,bias", [(4, 2, 16, 24, 16, True, True), (6, 3, 10, 5, 4, True, True), (3, 1, 7, 7, 6, False, True), (2, 2, 64, 64, 0, False, False), (8, 1, 128, 40, 64, True, True),
                                                      (40, 8, 128, 128, 128, True, True)])
def test_biased_half_split_rotary_into_pages(dev, H, G, D, Dv, dims, own_v, bias, dt):
    """queries and keys turn, values (of their own, or the keys before they turn) do not; everything in the right place of the right page, nothing else touched"""
    from mistralrs_amd.hybrid import _call
    _lib.load("hybrid")
    g = torch.Generator().manual_seed(D)
    TT, bs = (torch.float32, torch.bfloat16)[dt == 1], 4
    nq, nk, nv = H * D, G * D, G * Dv
    for T in (6, 300):
        pos = torch.randint(0, 3000, (T,), generator=g).to(torch.int32)
        slots = torch.randperm(2 * T, generator=g)[:T]
        slots[1] = -1                                   # a row without a page
        blocks = -(-2 * T // bs)
        u = torch.randn(T, nq + nk + (nv if own_v else 0) + 3, generator=g)
        qb, kb, vb = (torch.randn(n, generator=g) if bias else torch.zeros(n) for n in (nq, nk, nv))
        if not own_v:
            vb = kb
        rot = {"dims": dims, "base": 50.0, "scaling": {"factor": 4.0, "fast": 2.0, "slow": 0.5, "original": 100}}
        f, mult = O.frequencies(rot) if dims else ([0.0], 1.0)
        q = torch.empty(T, nq, dtype=TT, device=dev)
        kc, vc = torch.full((blocks, G, bs, D), 9.0, dtype=TT, device=dev), torch.full((blocks, G, bs, Dv), 9.0, dtype=TT, device=dev)
        d = lambda t: t.to(dev) if bias else None
        _call("mrs_hyb_rope_half_cache", u.to(dev), u.shape[1], nq + nk if own_v else nq, d(qb), d(kb), d(vb), torch.tensor(f).float().to(dev), mult, pos.to(dev), slots.to(dev), q, kc, vc, T, H, G,
              D, Dv, dims, bs, dt)
        ud = u.double()
        bar = 2e-6 if dt == 2 else 4e-3
        fp = torch.tensor(f).float().double()          # the angles the kernel sees: f32 products
        ang = (pos.float()[:, None] * fp.float()).double()[:, None, :]

        def turn(x):
            h = dims // 2
            c, s = torch.cos(ang) * mult, torch.sin(ang) * mult
            return torch.cat([x[..., :h] * c - x[..., h:2 * h] * s, x[..., h:2 * h] * c + x[..., :h] * s, x[..., 2 * h:]], -1) if dims else x
        qw = turn((ud[:, :nq] + qb.double()).view(T, H, D))
        kr = (ud[:, nq:nq + nk] + kb.double()).view(T, G, D)
        vw = (ud[:, nq + nk:nq + nk + nv] + vb.double()).view(T, G, Dv) if own_v else kr
        assert rel(q.double().cpu().view(T, H, D), qw) < bar
        kc, vc = kc.double().cpu().transpose(1, 2).reshape(-1, G, D), vc.double().cpu().transpose(1, 2).reshape(-1, G, Dv)
        on = slots >= 0
        assert rel(kc[slots[on]], turn(kr)[on]) < bar and rel(vc[slots[on]], vw[on]) < bar
        rest = torch.ones(len(kc), dtype=torch.bool)
        rest[slots[on]] = False
        assert bool((kc[rest] == 9).all()) and bool((vc[rest] == 9).all())


# ---- attention over pages
def pages_of(k, v, bs, dev, dtype, seed, extra=3):
    """keys and values [N, G, D] of several sequences in shuffled pages; slots without a token hold NaN.  Returns (k_cache, v_cache, block lists, number of blocks)"""
    g = torch.Generator().manual_seed(seed)
    need = [-(-len(x) // bs) for x in k]
    order = torch.randperm(sum(need) + extra, generator=g).tolist()
    G, D, Dv = k[0].shape[1], k[0].shape[2], v[0].shape[2]
    kc, vc = torch.full((len(order), G, bs, D), float("nan")), torch.full((len(order), G, bs, Dv), float("nan"))
    lists = []
    for kk, vv, n in zip(k, v, need):
        blk, order = order[:n], order[n:]
        lists.append(blk)
        for j in range(len(kk)):
            kc[blk[j // bs], :, j % bs], vc[blk[j // bs], :, j % bs] = kk[j], vv[j]
    return kc.to(dev, dtype), vc.to(dev, dtype), lists, kc.shape[0]


def reference(q, k, v, p0, scale, lo_of, sink=None, gate=None):
    """q [T, H, D] at p0 ..; k / v [N, G, *]; lo_of(i): the positions j <= i that i sees"""
    T, H, _ = q.shape
    out = torch.zeros(T, H, v.shape[2], dtype=D64)
    for t in range(T):
        see = lo_of(p0 + t)
        for h in range(H):
            g = h // (H // k.shape[1])
            s = (k[see, g] @ q[t, h]) * scale
            if sink is not None:
                s = torch.cat([s, sink[h:h + 1]])
            p = torch.softmax(s, 0)[:len(see)]
            out[t, h] = p @ v[see, g]
    return out if gate is None else out * torch.sigmoid(gate)[:, :, None]


VIEWS = {"chunk_8": dict(chunk=8), "chunk_33": dict(chunk=33), "chunk_64": dict(chunk=64), "window_7": dict(window=7), "window_64": dict(window=64), "all": {}}


def sees(chunk=0, window=0):
    return lambda i: list(range((i // chunk) * chunk if chunk else max(0, i - window + 1) if window else 0, i + 1))


@pytest.mark.gpu
@pytest.mark.parametrize("view", sorted(VIEWS))
@pytest.mark.parametrize("form", ["matrix_cores", "general_bf16", "general_f32"])
@pytest.mark.parametrize("H,G,D,Dv,bs", [(4, 2, 16, 24, 8), (3, 1, 88, 184, 12), (2, 2, 200, 256, 16), (6, 2, 128, 128, 32), (5, 5, 8, 8, 5)])
def test_paged_attention_over_portions_and_single_rows(dev, H, G, D, Dv, bs, form, view):
    """portions (down to one row) and single rows of several sequences over shuffled pages; one key per sequence stands out, one lies just outside what most rows see, so that a key too
    many or too few is an error of the size of the values; learned sinks and a gate per head"""
    from mistralrs_amd.hybrid import RaggedBatch, _call
    _lib.load("hybrid")
    g = torch.Generator().manual_seed(D + bs)
    opt = VIEWS[view]
    TT, dt = (torch.float32, 2) if form == "general_f32" else (torch.bfloat16, 1)
    ents = [(0, 70), (37, 29), (64, 1), (100, 40), (9, 2)]
    k, v, q = [], [], []
    for p0, n in ents:
        N = p0 + n
        kk, vv, qq = torch.randn(N, G, D, generator=g), torch.randn(N, G, Dv, generator=g), torch.randn(n, H, D, generator=g)
        kk[max(0, N - 12)] *= 3.0                          # stands out for the queries it agrees with
        edge = opt.get("chunk") or opt.get("window")
        if edge and N > edge:                              # in front of the edge of the last row: would take nearly all the weight of every row that must not see it
            last = N - 1
            j = (last // edge) * edge - 1 if "chunk" in opt else last - edge
            if j >= 0:
                kk[j] = 8.0 * qq[-1].view(G, H // G, D).mean(1)
        k.append(kk.to(TT)), v.append(vv.to(TT)), q.append(qq.to(TT))
    kc, vc, lists, nb = pages_of(k, v, bs, dev, TT, bs)
    sink, gate = torch.randn(H, generator=g), torch.randn(sum(n for _, n in ents), H, generator=g)
    for decode in (False, True):
        if decode:
            rows = [(p0 + n - 1, 1) for p0, n in ents]
            qs = [x[-1:] for x in q]
            gt = gate[torch.tensor([sum(n for _, n in ents[:i + 1]) - 1 for i in range(len(ents))])]
        else:
            rows, qs, gt = ents, q, gate
        b = _batch(dev, [(p0, n, 0) for p0, n in rows], bs, lists)
        T = b.rows
        out = torch.empty(T, H * Dv, dtype=TT, device=dev)
        seg = (b.seg_entry, b.seg_row0, b.seg_len, b.segments, RaggedBatch.SEGMENT)
        qd, sd, gd = torch.cat(qs).reshape(T, H * D).to(dev), sink.to(dev), gt.to(dev).contiguous()
        if form == "matrix_cores":
            _call("mrs_hyb_attn_mfma_prompt", qd, kc, vc, b.block_tables, b.tok_pos, *seg, sd, gd, H, 0, out, T, H, G, D, Dv, nb, b.max_blocks, bs, opt.get("window", 0), opt.get("chunk", 0), D ** -0.5)
        elif "window" in opt:
            ge = gd[:, :, None].expand(T, H, Dv).reshape(T, H * Dv).contiguous()
            _call("mrs_hyb_paged_attn_sink_window", qd, kc, vc, b.block_tables, b.tok_seq, b.tok_pos, out, T, H, G, D, Dv, bs, b.max_blocks, opt["window"], 0, D ** -0.5, dt, *seg, 0.0, 1, sd, ge, H * Dv,
                  None, 0, 0, 0)
        else:
            sp = 2 if decode else 0
            scratch = torch.empty(2, T, H, Dv + 2, device=dev) if decode else None
            _call("mrs_hyb_paged_attn_chunked", qd, kc, vc, b.block_tables, b.tok_seq, b.tok_pos, out, T, H, G, D, Dv, bs, b.max_blocks, opt.get("chunk", 0), D ** -0.5, dt, *seg, 0.0, 1, sd, gd, H, 1,
                  scratch, sp)
        at = 0
        for (p0, n), qq, kk, vv in zip(rows, qs, k, v):
            want = reference(qq.double(), kk.double(), vv.double(), p0, D ** -0.5, sees(**opt), sink.double(), gt.double()[at:at + n]).reshape(n, H * Dv)
            got = out[at:at + n].double().cpu()
            assert float((got - want).abs().max()) < (3e-5 if dt == 2 else 1.5e-2 * float(want.abs().max())), (decode, p0)
            at += n


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H,G,D,Dv", [(1, 1, 16, 16), (8, 8, 64, 64), (6, 2, 24, 10), (10, 2, 128, 130), (16, 2, 64, 256), (48, 3, 40, 300), (12, 1, 576, 512), (9, 3, 7, 5), (2, 1, 16, 9)])
def test_single_rows_whose_query_heads_share_keys(dev, H, G, D, Dv, dtype):
    """groups of 1 .. 16 query heads per key head, long contexts dealt to workgroups or not, kept first tokens, windows, capped scores"""
    from mistralrs_amd.hybrid import RaggedBatch, _call
    _lib.load("hybrid")
    g = torch.Generator().manual_seed(H + D)
    TT, dt = (torch.float32, 2) if dtype == "float32" else (torch.bfloat16, 1)
    lens, bs = [300, 1, 67], 16
    k = [torch.randn(n, G, D, generator=g).to(TT) for n in lens]
    v = [torch.randn(n, G, Dv, generator=g).to(TT) for n in lens]
    q = torch.randn(3, H, D, generator=g).to(TT)
    kc, vc, lists, _ = pages_of(k, v, bs, dev, TT, 3)
    b = _batch(dev, [(n - 1, 1, 0) for n in lens], bs, lists)
    seg = (b.seg_entry, b.seg_row0, b.seg_len, b.segments, RaggedBatch.SEGMENT)
    for window, keep, cap, splits in ((0, 0, 0.0, 0), (0, 0, 0.0, 3), (50, 5, 0.0, 0), (40, 0, 2.0, 2), (0, 0, 5.0, 7)):
        out = torch.empty(3, H * Dv, dtype=TT, device=dev)
        scratch = torch.full((splits, 3, H, Dv + 2), float("nan"), device=dev) if splits else None
        _call("mrs_hyb_paged_attn_opts", q.reshape(3, -1).to(dev), kc, vc, b.block_tables, b.tok_seq, b.tok_pos, out, 3, H, G, D, Dv, bs, b.max_blocks, window, keep, D ** -0.5, dt, *seg, cap, 0, None, 0,
              scratch, splits, 0)
        for e, n in enumerate(lens):
            see = [j for j in range(n) if not window or n - 1 - j < window or j < keep]
            want = torch.zeros(H, Dv, dtype=D64)
            for h in range(H):
                s = (k[e].double()[see, h // (H // G)] @ q[e, h].double()) * D ** -0.5
                s = cap * torch.tanh(s / cap) if cap else s
                want[h] = torch.softmax(s, 0) @ v[e].double()[see, h // (H // G)]
            assert rel(out[e].double().cpu().view(H, Dv), want) < (5e-6 if dt == 2 else 5e-3), (window, keep, cap, splits, e)


@pytest.mark.gpu
@pytest.mark.parametrize("form", ["portions", "single_rows"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("chunk", [8, 20, 64, 100])
def test_planted_keys_at_the_chunk_edges(dev, chunk, dtype, form):
    """position i's query matches ONE key; the value there spells its position: read back when the key lies inside the chunk (its first position, the query itself, both sides of a page
    border), near-uniform weights without it when the key is the last one of the chunk before"""
    from mistralrs_amd.hybrid import RaggedBatch, _call
    _lib.load("hybrid")
    TT, dt = (torch.float32, 2) if dtype == "float32" else (torch.bfloat16, 1)
    N, H, G, D, Dv, bs = 230, 2, 1, 256, 16, 16
    g = torch.Generator().manual_seed(chunk)
    code = torch.sign(torch.randn(N, D, generator=g))                        # nearly orthogonal codes: a query carries the code of the key it looks for
    v = (torch.arange(N)[:, None] >> torch.arange(Dv)[None, :] & 1).float() * 2 - 1
    k = code.view(N, 1, D)
    asked = []
    for i in range(N):
        start = (i // chunk) * chunk
        asked.append([start, i, start - 1, max(start, (i // bs) * bs), max(start, (i // bs) * bs - 1)][i % 5])
    q = torch.stack([code[max(0, j)] for j in asked]).view(N, 1, D).expand(N, H, D)
    kc, vc, lists, nb = pages_of([k.to(TT)], [v.view(N, 1, Dv).to(TT)], bs, dev, TT, 1)
    out = torch.empty(N, H * Dv, dtype=TT, device=dev)
    cuts = [(0, 2), (2, 63), (65, 1), (66, 100), (166, 64)] if form == "portions" else [(i, 1) for i in range(N)]
    scale = 0.25
    for p0, n in cuts:
        b = _batch(dev, [(p0, n, 0)], bs, lists)
        seg = (b.seg_entry, b.seg_row0, b.seg_len, b.segments, RaggedBatch.SEGMENT)
        qd = q[p0:p0 + n].reshape(n, H * D).to(dev, TT).contiguous()
        if dt == 1 and n > 1:
            _call("mrs_hyb_attn_mfma_prompt", qd, kc, vc, b.block_tables, b.tok_pos, *seg, None, None, 0, 0, out[p0:], n, H, G, D, Dv, nb, b.max_blocks, bs, 0, chunk, scale)
        else:
            _call("mrs_hyb_paged_attn_chunked", qd, kc, vc, b.block_tables, b.tok_seq, b.tok_pos, out[p0:], n, H, G, D, Dv, bs, b.max_blocks, chunk, scale, dt, *seg, 0.0, 0, None, None, 0, 0, None, 0)
    got = out.float().cpu().view(N, H, Dv)
    for i in range(N):
        j, start = asked[i], (i // chunk) * chunk
        for h in range(H):
            if j >= start:
                assert torch.allclose(got[i, h], v[j], atol=1e-2), (i, j)
            else:
                see = k[start:i + 1, 0].double() @ q[i, h].double() * scale
                want = torch.softmax(see, 0) @ v[start:i + 1].double()
                assert torch.allclose(got[i, h].double(), want, atol=1e-2), (i, j)


@pytest.mark.gpu
def test_matrix_core_weights_keep_their_low_bits(dev):
    """two keys of opposite values whose weights differ by a few parts in 2^20: the difference survives only if the weights enter the value product as f32 numbers"""
    from mistralrs_amd.hybrid import RaggedBatch, _call
    _lib.load("hybrid")
    N, D, Dv, bs = 64, 16, 8, 16
    k, v = torch.zeros(N, 1, D), torch.zeros(N, 1, Dv)
    k[:, 0, 0], k[10, 0, 1] = -60.0, 2.0 ** -8
    k[10, 0, 0] = k[40, 0, 0] = 0.0
    v[10], v[40] = 1.0, -1.0
    q = torch.zeros(2, 1, D)
    q[:, 0, 0], q[:, 0, 1] = 1.0, 2.0 ** -8
    kc, vc, lists, nb = pages_of([k.to(torch.bfloat16)], [v.to(torch.bfloat16)], bs, dev, torch.bfloat16, 2)
    b = _batch(dev, [(62, 2, 0)], bs, lists)
    out = torch.empty(2, Dv, dtype=torch.bfloat16, device=dev)
    _call("mrs_hyb_attn_mfma_prompt", q.view(2, D).to(dev, torch.bfloat16), kc, vc, b.block_tables, b.tok_pos, b.seg_entry, b.seg_row0, b.seg_len, b.segments, RaggedBatch.SEGMENT, None, None, 0, 0, out, 2,
          1, 1, D, Dv, nb, b.max_blocks, bs, 0, 0, 1.0)
    want = math.tanh(2.0 ** -16 / 2)
    assert torch.allclose(out.float().cpu(), torch.full((2, Dv), want), rtol=0.02, atol=0)


# ---- recurrences
RAGGED = [[(0, 130, 2), (0, 1, 0), (0, 64, 3), (0, 7, 1)], [(130, 1, 2), (1, 70, 0), (64, 2, 3), (7, 65, 1)], [(131, 1, 2), (71, 1, 0), (66, 1, 3), (72, 1, 1)], [(132, 3, 2), (0, 200, 0), (67, 1, 3), (73, 1, 1)]]


def run_ragged(dev, make, call, cell, slots=4):
    """steps of portions and single rows through slots that held NaN or huge numbers before: `make(rows)` draws a request's inputs, `call(batch, inputs)` runs the kernels on the rows of a
    step, `cell(inputs, state)` restates one request's rows"""
    state, reqs = {}, {}
    for step in RAGGED:
        ins, want = [], []
        for p0, n, slot in step:
            if p0 == 0:
                state[slot] = None
            x = make(n)
            ins.append(x)
            o, state[slot] = cell(x, state[slot])
            want.append(o)
        b = _batch(dev, step)
        single = b.seg_rows == 1
        got = call(b, [torch.cat(t) for t in zip(*ins)], single)
        at = 0
        for (p0, n, _), w in zip(step, want):
            yield got[at:at + n].double().cpu(), w, (p0, n)
            at += n


def segment_table(b, seg):
    if not seg:
        return b.entry_table(), b.entries
    *table, n = b.segment_table(seg)
    return table, n


@pytest.mark.gpu
@pytest.mark.parametrize("seg", [0, 32, 64], ids=["chains", "segments_of_32", "segments_of_64"])
@pytest.mark.parametrize("H,D,Dv", [(3, 16, 8), (2, 32, 32), (2, 64, 16), (3, 7, 5), (1, 130, 3), (2, 128, 260), (5, 1, 1), (1, 300, 70), (1, 48, 130)])
def test_decayed_linear_attention_over_portions_single_rows_and_reused_slots(dev, H, D, Dv, seg):
    from mistralrs_amd.hybrid import _call
    _lib.load("hybrid")
    g = torch.Generator().manual_seed(D + Dv)
    decay = torch.tensor([[0.5, 0.9, 0.999, 1.0, 0.25][h % 5] for h in range(H)])
    st = torch.full((4, H, D, Dv), float("nan"), device=dev)
    st[1] = 1e6
    nk, nv = H * D, H * Dv

    def call(b, x, single):
        T, u = b.rows, x[0].to(dev)
        y = torch.empty(T, nv, device=dev)
        if single:
            _call("mrs_hyb_lightning_step", u, u.stride(0), nv, nv + nk, decay.to(dev), st, y, b.seq_start, b.seq_pos0, b.seq_slot, T, b.entries, H, D, Dv)
        else:
            table, n = segment_table(b, seg)
            carry, dec = torch.empty(n, H, D, Dv, device=dev), torch.empty(n, H, D, device=dev)
            _call("mrs_hyb_lightning_scan", u, u.stride(0), nv, nv + nk, decay.to(dev), st, y, b.seq_pos0, b.seq_slot, *table, carry, dec, T, b.entries, n, H, D, Dv)
        return y

    def cell(x, S):
        u = O.silu(x[0].double())
        n = len(u)
        o, S = O.decayed_cell(u[:, nv + nk:nv + 2 * nk].view(n, H, D), u[:, nv:nv + nk].view(n, H, D), u[:, :nv].view(n, H, Dv), decay.double(), S if S is not None else torch.zeros(H, D, Dv, dtype=D64))
        return o.reshape(n, nv), S
    for got, want, at in run_ragged(dev, lambda n: (torch.randn(n, nv + 2 * nk + 4, generator=g) * 1.5,), call, cell):
        assert rel(got, want) < 5e-6, at


@pytest.mark.gpu
@pytest.mark.parametrize("dt", [2, 1], ids=["f32", "bf16"])
@pytest.mark.parametrize("seg", [0, 32, 64], ids=["chains", "segments_of_32", "segments_of_64"])
@pytest.mark.parametrize("H,D,rank", [(3, 16, 5), (2, 32, 16), (2, 64, 1), (3, 7, 3), (1, 130, 40), (5, 1, 2), (1, 256, 8)])
def test_time_mixing_recurrence_over_portions_single_rows_and_reused_slots(dev, H, D, rank, seg, dt):
    """decays from the two-step projection, the read-out before the update plus the bonus, head norm with a full weight, gate"""
    from mistralrs_amd.hybrid import _call
    _lib.load("hybrid")
    g = torch.Generator().manual_seed(D)
    TT = torch.float32 if dt == 2 else torch.bfloat16
    n = H * D
    w2, w0, bonus, norm = (torch.randn(n, rank, generator=g) * rank ** -0.5).to(TT), torch.randn(n, generator=g) - 1.0, torch.randn(H, D, generator=g), torch.randn(n, generator=g)
    st = torch.full((4, H, D, D), float("nan"), device=dev)
    st[1] = 1e6
    dv = lambda t: t.to(dev)

    def call(b, x, single):
        T, u, a1 = b.rows, dv(x[0]), dv(x[1])
        o = torch.empty(T, n, dtype=TT, device=dev)
        if single:
            _call("mrs_hyb_bonus_step", u, u.stride(0), n, 2 * n, 3 * n, a1, rank, dv(w2), dv(w0), dv(bonus), dv(norm), st, o, b.seq_start, b.seq_pos0, b.seq_slot, T, b.entries, H, D, D, 1e-5, dt)
            return o
        t1, z, y = torch.empty(T, rank, dtype=TT, device=dev), torch.empty(T, n, device=dev), torch.empty(T, n, device=dev)
        _call("mrs_hyb_tanh_round", a1, t1, T, rank, dt)
        assert torch.allclose(t1.float(), torch.tanh(a1), atol=4e-3 if dt == 1 else 1e-6)
        z.copy_(dv(t1.double().cpu() @ w2.double().T))
        _call("mrs_hyb_gla_decays", z, dv(w0), T, n, 0.0)
        table, ns = segment_table(b, seg)
        carry, dec = torch.empty(ns, H, D, D, device=dev), torch.empty(ns, H, D, device=dev)
        _call("mrs_hyb_bonus_scan", u, u.stride(0), n, 2 * n, z, dv(bonus), st, y, b.seq_pos0, b.seq_slot, *table, carry, dec, T, b.entries, ns, H, D, D)
        _call("mrs_hyb_head_norm_gate", y, D, None, dv(norm), 1, u[:, 3 * n:], u.stride(0), 2, o, T, H, D, 1e-5, dt)
        return o

    def cell(x, S):
        u, m = x[0].double(), len(x[0])
        r = torch.tanh(x[1].double()).to(TT).double()
        v, k, q = (u[:, i * n:(i + 1) * n].view(m, H, D) for i in range(3))
        o, S = O.bonus_cell(q, k, v, torch.exp(-torch.exp(r @ w2.double().T + w0.double())).view(m, H, D), bonus.double(), S if S is not None else torch.zeros(H, D, D, dtype=D64))
        return O.rms_norm(o, 1.0, 1e-5).reshape(m, n) * norm.double() * O.silu(u[:, 3 * n:4 * n]), S
    for got, want, at in run_ragged(dev, lambda m: (torch.randn(m, 4 * n + 4, generator=g), torch.randn(m, rank, generator=g)), call, cell):
        assert rel(got, want) < (1e-5 if dt == 2 else 6e-3), at


@pytest.mark.gpu
@pytest.mark.parametrize("dt", [2, 1], ids=["f32", "bf16"])
@pytest.mark.parametrize("C,blocks", [(48, 3), (40, 1), (144, 2), (7, 7), (15, 3), (260, 2), (192, 1), (1, 1), (1024, 4)])
def test_gated_recurrent_unit_over_portions_single_rows_and_reused_slots(dev, C, blocks, dt):
    """gates of channel parts of many sizes, segments and their carry, the GELU branch; log a from nearly zero to far below: states that keep and states that forget"""
    from mistralrs_amd.hybrid import _call
    _lib.load("hybrid")
    g = torch.Generator().manual_seed(C)
    TT, part = (torch.float32, C // blocks) if dt == 2 else (torch.bfloat16, C // blocks)
    wa, wi = ((torch.randn(blocks, part, part, generator=g) * part ** -0.5).to(torch.bfloat16) for _ in range(2))
    ba, bi, yb = (torch.randn(C, generator=g) for _ in range(3))
    lam = torch.linspace(-9, 2, C)
    st = torch.full((4, C), float("nan"), device=dev)
    st[1] = 1e6
    dv = lambda t: t.to(dev)

    def call(b, x, single):
        T, u, y = b.rows, dv(x[0]), dv(x[1])
        o = torch.empty(T, C, dtype=TT, device=dev)
        gates = (dv(wa.to(TT)), dv(wi.to(TT)), dv(ba), dv(bi), dv(lam), y, y.stride(0), dv(yb), st)
        if single:
            _call("mrs_hyb_rglru_step", u, *gates, o, b.seq_start, b.seq_pos0, b.seq_slot, T, b.entries, C, blocks, dt)
        else:
            loc, prod, start = torch.empty(T, C, device=dev), torch.empty(T, C, device=dev), torch.empty(b.segments, C, device=dev)
            _call("mrs_hyb_rglru_scan", u, *gates, loc, prod, start, o, b.seq_pos0, b.seq_slot, b.seg_row0, b.seg_len, b.ent_seg0, T, b.entries, b.segments, 64, C, blocks, dt)
        return o

    def cell(x, S):
        u = x[0].double()
        r, i = O.block_gate(u, wa.double(), ba.double().view(blocks, part)), O.block_gate(u, wi.double(), bi.double().view(blocks, part))
        s, S = O.rglru_cell(u, r, i, lam.double(), S if S is not None else torch.zeros(C, dtype=D64))
        return s * O.gelu_tanh(x[1].double()[:, :C] + yb.double()), S
    for got, want, at in run_ragged(dev, lambda n: (torch.randn(n, C, generator=g), torch.randn(n, 2 * C, generator=g)), call, cell):
        assert rel(got, want) < (5e-6 if dt == 2 else 4e-3), at


@pytest.mark.gpu
@pytest.mark.parametrize("W", [40, 7, 600])
def test_token_shift_reads_the_row_before_across_steps(dev, W):
    from mistralrs_amd.hybrid import _call
    _lib.load("hybrid")
    g = torch.Generator().manual_seed(W)
    mu = torch.randn(5, W, generator=g)
    last = torch.full((4, W), float("nan"), device=dev)
    for dt, TT in ((2, torch.float32), (1, torch.bfloat16)):
        def call(b, x, single):
            out = torch.empty(5, b.rows, W, dtype=TT, device=dev)
            _call("mrs_hyb_token_shift", x[0].to(dev), mu.to(dev), last, out, b.tok_seq, b.seq_start, b.seq_pos0, b.seq_slot, b.rows, W, 5, dt)
            return out.transpose(0, 1).reshape(b.rows, 5 * W)

        def cell(x, st):
            h = x[0].double()
            p = O.shifted(h, st)
            return torch.cat([h + (p - h) * m for m in mu.double()], -1), h[-1]
        for got, want, at in run_ragged(dev, lambda n: (torch.randn(n, W, generator=g),), call, cell):
            assert rel(got, want) < (1e-6 if dt == 2 else 4e-3), at


# ---------------------------------------------------------------------------------------------------------------- mixers alone (GPU)
def mixer_alone(dev, layer, dtype, bar, seed, cuts=(2, 61, 1, 1, 70, 1, 5), rank=5):
    """one mixer of one layer: its output rows (no stream, no norm) in portions and single rows against the restatement's whole prompt"""
    from mistralrs_amd.hybrid import HybridCache, HybridDecoder, RaggedBatch, zumuzen_spec
    cfg = config([layer])
    w = weights(cfg, seed, rank=rank)
    m = HybridDecoder(zumuzen_spec(cfg), dev, dtype, num_blocks=24, block_size=16, state_slots=2)
    m.load_weights(w.__getitem__)
    cache, mx = HybridCache(m), m.layers[0].mixer
    h = torch.randn(sum(cuts), cfg["width"], generator=torch.Generator().manual_seed(seed + 1)).to(torch.bfloat16)
    want, _ = O.mixer(h.double(), layer, f64(w), "l0.mix.", cfg["norm"]["eps"], None, 0)
    got, at = [], 0
    for n in cuts:
        assert cache.reserve(7, at + n)
        b = RaggedBatch.build([cache.entry(7, [0] * n, at)], 16, dev)
        x = torch.full((n, cfg["width"]), 2.0, device=dev)
        hd = h[at:at + n].to(dev, m.torch_dtype).contiguous()
        mx.forward(hd, x, b, accumulate=at % 2 == 0, **({"h32": hd.float()} if mx.wants_f32_input else {}))
        got.append(x.double().cpu() - (2.0 if at % 2 == 0 else 0.0))
        at += n
    assert close(torch.cat(got), want, bar)


@pytest.mark.gpu
@BOTH
@pytest.mark.parametrize("kw", [dict(), dict(width=40, blocks=1, conv=1), dict(width=7, blocks=7, conv=3), dict(width=130, blocks=2, conv=9), dict(width=256, blocks=2, conv=2)])
def test_recurrent_block_alone(dev, kw, dtype, bar):
    mixer_alone(dev, lru(**kw), dtype, bar, 31)


@pytest.mark.gpu
@BOTH
@pytest.mark.parametrize("kw", [dict(), dict(heads=6, kv=1, dim=24, vdim=8, dims=6, size=7), dict(heads=1, kv=1, dim=2, vdim=1, dims=2, size=1, l_heads=1, l_dim=1, l_vdim=1), dict(dim=64, vdim=96, dims=32, size=64,
                                l_heads=2, l_dim=64, l_vdim=130), dict(heads=3, kv=3, dim=10, vdim=7, dims=4, size=33, l_heads=5, l_dim=7, l_vdim=3), dict(size=0)])
def test_attention_beside_decayed_linear_attention_alone(dev, kw, dtype, bar):
    mixer_alone(dev, par(**kw), dtype, bar, 32)


@pytest.mark.gpu
@BOTH
@pytest.mark.parametrize("kw", [dict(), dict(heads=6, kv=1, dim=24, dims=6, size=7), dict(heads=1, kv=1, dim=2, dims=2, size=1, t_heads=1, t_dim=1, ls=1.0, rs=1.0), dict(dim=64, dims=64, size=64, t_heads=2, t_dim=64),
                                dict(heads=3, kv=3, dim=10, dims=4, size=33, t_heads=5, t_dim=7, scaling=None, ls=-0.5), dict(size=0, rs=2.0)])
def test_keys_as_values_beside_time_mixing_alone(dev, kw, dtype, bar):
    mixer_alone(dev, par2(**kw), dtype, bar, 33, rank=1 if kw.get("t_dim") == 1 else 5)


@pytest.mark.gpu
@BOTH
def test_sharp_attention_needs_the_chunk_the_sink_the_ramp_and_the_biases(dev, dtype, bar):
    """scores large enough that single keys dominate: the served model follows the restatement, and a restatement without the chunk's edge, the sink, the ramp, the biases, the unrotated
    values, the bonus or the passes' vectors is far away"""
    cfg = config([par2(scale=1.0, size=24), par(scale=1.0, size=17)], loop=(0, 2, 2))
    w = weights(cfg, 8)
    w["l0.mix.left.sink"] = w["l0.mix.left.sink"] + 3
    w["l1.mix.left.v.b"] = w["l1.mix.left.v.b"] * 4
    t = toks(80, cfg["vocab"], 16)
    want = logits_of(cfg, f64(w), t)
    sv = Served(cfg, w, dev, dtype)
    got = torch.cat(sv.step([(1, t[:47])]) + sv.step([(1, t[47:70])]) + [sv.step([(1, [x])])[0] for x in t[70:]])
    assert close(got, want, 2 * bar)

    def changed(edit_cfg=None, edit_w=None):
        c = json.loads(json.dumps(cfg))
        x = {k: v.clone() for k, v in w.items()}
        if edit_cfg:
            edit_cfg(c)
        if edit_w:
            edit_w(x)
        return rel(logits_of(c, f64(x), t), want)
    left = lambda c, i: c["layers"][i]["mixer"]["left"]
    far = {"chunk": changed(lambda c: left(c, 0)["mask"].update(size=25)), "chunk_b": changed(lambda c: left(c, 1)["mask"].update(size=9)),
           "ramp": changed(lambda c: left(c, 0)["rot"].pop("scaling")), "sink": changed(None, lambda x: x["l0.mix.left.sink"].fill_(-1e4)),
           "bias": changed(None, lambda x: x["l0.mix.left.k.b"].zero_()), "v_bias": changed(None, lambda x: x["l1.mix.left.v.b"].zero_()), "bonus": changed(None, lambda x: x["l0.mix.right.u"].zero_()),
           "shift": changed(None, lambda x: x["l0.mix.right.mu.k"].zero_()), "step": changed(None, lambda x: x["loop.step"].copy_(x["loop.step"].flip(0))),
           "scale": changed(lambda c: c["layers"][0]["mixer"].update(right_scale=0.7, left_scale=1.3)), "decay": changed(lambda c: c["layers"][1]["mixer"]["right"].update(decay=[0.5, 0.5, 0.5]))}
    assert min(far.values()) > (20 if dtype == "float32" else 2) * 2 * bar, far


@pytest.mark.gpu
def test_slow_decays_carry_the_first_tokens_across_a_long_prompt_and_decoding(dev):
    """states that forget slowly: two prompts that differ in their first token only stay apart by more than rounding 400 rows later, and the served model agrees with the restatement"""
    cfg = config([lru(), par2(size=8), par(size=8, decay=[1.0, 0.9999, 0.999])], loop=(1, 3, 2))
    w = weights(cfg, 21, slow=True)
    wd = f64(w)
    t = toks(420, cfg["vocab"], 22)
    other = [(t[0] + 1) % cfg["vocab"]] + t[1:]
    want, alt = logits_of(cfg, wd, t), logits_of(cfg, wd, other)
    assert rel(want[-20:], alt[-20:]) > 2e-3
    sv = Served(cfg, w, dev, max_tokens=1024)
    got = torch.cat(sv.step([(1, t[:300])]) + sv.step([(1, t[300:390])]) + [sv.step([(1, [x])])[0] for x in t[390:]])
    assert rel(got, want) < 5e-5 and rel(got[-20:], want[-20:]) < 0.05 * rel(want[-20:], alt[-20:])


@pytest.mark.gpu
@BOTH
@pytest.mark.parametrize("size", [0, 600, 300, 70])
def test_long_decoding_with_keys_dealt_to_several_workgroups(dev, size, dtype, bar):
    """decoding across chunk edges with contexts long enough that the keys of a row go to several workgroups"""
    cfg = config([par(size=size, mlp=None), par2(size=size, mlp=None)])
    w = weights(cfg, 23)
    t = toks(640, cfg["vocab"], 24)
    want = logits_of(cfg, f64(w), t)
    sv = Served(cfg, w, dev, dtype, max_tokens=1400)
    assert close(sv.step([(1, t[:570])])[0], want[:570], bar)
    sv.step([(2, t[:590])])
    got = {1: [], 2: []}
    for i in range(50):
        o = sv.step([(1, [t[570 + i]]), (2, [t[590 + i]])])
        got[1].append(o[0])
        got[2].append(o[1])
    assert close(torch.cat(got[1]), want[570:620], bar) and close(torch.cat(got[2]), want[590:640], bar)


@pytest.mark.gpu
def test_first_tokens_see_zeros_not_the_slots_former_owner(dev):
    cfg = config(STACK, loop=LOOP)
    w = weights(cfg, 25)
    wd = f64(w)
    sv = Served(cfg, w, dev, slots=1, max_tokens=128)
    a, b = toks(90, cfg["vocab"], 26), toks(30, cfg["vocab"], 27)
    sv.step([(1, a)])
    sv.end(1)
    want = logits_of(cfg, wd, b)
    got = [sv.step([(2, [x])])[0] for x in b[:5]] + sv.step([(2, b[5:])])
    assert rel(torch.cat(got), want) < 5e-5
    sv.end(2)
    assert rel(sv.step([(3, b[:2])])[0], want[:2]) < 5e-5


# ---------------------------------------------------------------------------------------------------------------- whole models (GPU)
@pytest.mark.gpu
@BOTH
def test_whole_prompt_every_layer_run(dev, dtype, bar):
    cfg = config(STACK, loop=LOOP)
    w = weights(cfg, 5)
    sv = Served(cfg, w, dev, dtype)
    t = toks(150, cfg["vocab"], 14)
    want, after, _ = O.forward(cfg, f64(w), t)
    sv.m.trace_layers = []
    got = sv.step([(1, t)])[0]
    assert len(sv.m.trace_layers) == len(STACK) + 6 and sv.m.has_recurrent_state and sv.m.has_paged_kv
    assert sv.m.layers[4].mixer.conv_state is not sv.m.layers[1].mixer.conv_state and sv.m.layers[4].mixer.w_in is sv.m.layers[1].mixer.w_in
    for i, (a, b) in enumerate(zip(sv.m.trace_layers, after)):
        assert close(a.double().cpu(), b, bar), f"residual stream after layer run {i}"
    assert close(got, want, bar)


@pytest.mark.gpu
@BOTH
@pytest.mark.parametrize("loop", [None, (0, 6, 1), (5, 6, 2), (0, 2, 2), LOOP])
def test_portions_and_decoding_equal_the_whole_prompt(dev, loop, dtype, bar):
    """the same 200 tokens: whole; in portions of changing sizes down to two tokens and single tokens; token by token from the start"""
    cfg = config(STACK, loop=loop)
    w = weights(cfg, 6)
    t = toks(200, cfg["vocab"], 15)
    want = logits_of(cfg, f64(w), t)
    sv = Served(cfg, w, dev, dtype, max_tokens=640)
    assert close(sv.step([(1, t)])[0], want, bar)
    cuts = [2, 3, 1, 64, 2, 31, 1, 1, 65, 7, 2, 21]
    assert sum(cuts) == 200
    got, at = [], 0
    for c in cuts:
        got += sv.step([(2, t[at:at + c])])
        at += c
    assert close(torch.cat(got), want, bar)
    got = [sv.step([(3, [x])])[0] for x in t[:60]]
    assert close(torch.cat(got), want[:60], bar)


@pytest.mark.gpu
@BOTH
def test_mixed_batches_with_reused_pages_and_slots(dev, dtype, bar):
    """five requests of unequal length through a pool of 192 tokens and three slots: portions beside single tokens, a request left out of a step, pages and slots of finished
    requests taken by later ones -- every row against the request alone in the restatement"""
    cfg = config(STACK, loop=LOOP)
    w = weights(cfg, 7)
    wd = f64(w)
    sv = Served(cfg, w, dev, dtype, max_tokens=192, slots=3)
    req = {r: toks(n, cfg["vocab"], 20 + r) for r, n in ((1, 70), (2, 9), (3, 64), (4, 33), (5, 90))}
    full = {r: logits_of(cfg, wd, t) for r, t in req.items()}
    plan = [[(1, 40), (2, 1)], [(1, 1), (2, 3), (3, 33)], [(2, 5), (3, 1)], [(1, 29), (3, 30)], [(4, 2), (3, 0)], [(4, 31), (5, 60)], [(5, 1), (4, 0)], [(5, 29)]]
    at = {r: 0 for r in req}
    for step in plan:
        parts = [(r, req[r][at[r]:at[r] + n]) for r, n in step if n]
        outs = sv.step(parts)
        for (r, tk), o in zip(parts, outs):
            assert close(o, full[r][at[r]:at[r] + len(tk)], bar), (r, at[r])
            at[r] += len(tk)
            if at[r] == len(req[r]):
                sv.end(r)
    assert at == {r: len(t) for r, t in req.items()}


@pytest.mark.gpu
def test_sizes_that_coincide_or_equal_one(dev):
    """one head, chunks of one position, sizes equal to the width, scales of one, one-token prompts, a single pass, one tap"""
    for layers, kw in (([lru(width=24, blocks=1, conv=1, mlp=24), par(heads=1, kv=1, dim=24, vdim=24, dims=24, size=24, l_heads=1, l_dim=24, l_vdim=24, decay=[1.0], mlp=24),
                         par2(heads=1, kv=1, dim=24, dims=24, size=24, t_heads=1, t_dim=24, ls=1.0, rs=1.0, mlp=24)], dict(width=24, vocab=24, loop=(0, 3, 1))),
                       ([par2(heads=2, kv=1, dim=2, dims=2, size=1, t_heads=2, t_dim=1, mlp=1), lru(width=1, blocks=1, conv=2, mlp=None), par(heads=2, kv=2, dim=2, vdim=1, dims=2, size=2, l_heads=1, l_dim=1, l_vdim=1, mlp=None)],
                        dict(width=8, vocab=5, loop=(0, 1, 4)))):
        cfg = config(layers, **kw)
        w = weights(cfg, 9, rank=1)
        t = toks(40, cfg["vocab"], 17)
        want = logits_of(cfg, f64(w), t)
        sv = Served(cfg, w, dev)
        assert rel(sv.step([(1, t[:1])])[0], want[:1]) < 5e-5
        got = sv.step([(2, t[:1])]) + sv.step([(2, t[1:3])]) + sv.step([(2, t[3:])])
        assert rel(torch.cat(got), want) < 5e-5


@pytest.mark.gpu
@BOTH
def test_sizes_off_every_vector_width(dev, dtype, bar):
    """width, vocabulary, head sizes, ranks and feed-forward sizes that no 16-byte load divides: the element-wise paths of every kernel, prompt and decode"""
    cfg = config([lru(width=33, blocks=3, conv=5, mlp=27), par(heads=3, kv=3, dim=14, vdim=13, dims=6, size=11, l_heads=3, l_dim=11, l_vdim=13, mlp=15),
                  par2(heads=5, kv=1, dim=6, dims=2, size=37, t_heads=1, t_dim=33, mlp=9)], vocab=77, width=50, loop=(1, 3, 2))
    w = weights(cfg, 13, rank=3)
    t = toks(100, cfg["vocab"], 18)
    want = logits_of(cfg, f64(w), t)
    sv = Served(cfg, w, dev, dtype)
    got = sv.step([(1, t[:67])]) + sv.step([(1, t[67:90])]) + [sv.step([(1, [x])])[0] for x in t[90:]]
    assert close(torch.cat(got), want, bar)


@pytest.mark.gpu
@pytest.mark.parametrize("block_size", [8, 16, 12, 64])
def test_other_page_sizes(dev, block_size):
    cfg = config(STACK, loop=LOOP)
    w = weights(cfg, 16)
    t = toks(110, cfg["vocab"], 19)
    want = logits_of(cfg, f64(w), t)
    for dtype, bar in (("float32", 5e-5), ("bfloat16", 4e-2)):
        sv = Served(cfg, w, dev, dtype, block_size=block_size)
        got = sv.step([(1, t[:53])]) + sv.step([(1, t[53:100])]) + [sv.step([(1, [x])])[0] for x in t[100:]]
        assert close(torch.cat(got), want, bar), dtype


@pytest.mark.gpu
@pytest.mark.parametrize("graphs", [False, True], ids=["eager", "graphs"])
def test_greedy_generation_through_scheduler_and_engine(dev, graphs):
    """the package's own entry point: scheduler (pages + slots), engine, sampler; five prompts through three slots, against greedy decoding of the restatement"""
    from mistralrs_amd.cli import make_engine
    from mistralrs_amd.hybrid import HybridDecoder, zumuzen_spec
    from mistralrs_amd.sampler import SequenceSampler
    from mistralrs_amd.scheduler import Sequence
    cfg = config([lru(), par(), par2(size=9)], loop=(1, 3, 2))
    w = weights(cfg, 10)
    m = HybridDecoder(zumuzen_spec(cfg), dev, "float32", num_blocks=12, block_size=32, state_slots=3)
    m.load_weights(w.__getitem__)
    core = os.path.exists(_lib.path("core"))
    eng = make_engine(m, 12 * 32, 3, sampler=SequenceSampler(cfg["vocab"], dev, top_k=1) if core else None, max_batched_tokens=48, use_graphs=graphs)
    prompts = [toks(n, cfg["vocab"], 30 + n) for n in (5, 40, 1, 23, 60)]
    seqs = [Sequence(id=i + 1, tokens=list(p), max_new_tokens=6) for i, p in enumerate(prompts)]
    for s in seqs:
        eng.s.add_seq(s)
    eng.run()
    wd = f64(w)
    for p, s in zip(prompts, seqs):
        ref = list(p)
        for _ in range(6):
            lg = logits_of(cfg, wd, ref)[-1]
            top2 = torch.topk(lg, 2).values
            if float(top2[0] - top2[1]) < 1e-3:
                break  # a tie within rounding: the comparison stops here
            ref.append(int(lg.argmax()))
        assert s.error is None and s.generated[:len(ref) - len(p)] == ref[len(p):], (s.id, s.generated, ref[len(p):])
    assert eng.steps["prompt"] >= 2 and eng.steps["completion"] >= 6 and bool(eng._graphs) == graphs


@pytest.mark.gpu
@pytest.mark.parametrize("dtype,bar", [("float32", 1e-6), ("bfloat16", 2e-2)])
def test_captured_decode_steps_equal_eager_steps(dev, dtype, bar):
    """a HIP graph of one decode step for three sequences, captured while two of them are live: every replay (eager work and synchronisation between replays) against the
    eager step function on a second copy of the model, and the pages and slots the warm-up touched are intact"""
    cfg = config(STACK, loop=LOOP)
    w = weights(cfg, 11)
    a, b = Served(cfg, w, dev, dtype), Served(cfg, w, dev, dtype)
    prompts = {1: toks(37, cfg["vocab"], 41), 2: toks(3, cfg["vocab"], 42), 3: toks(64, cfg["vocab"], 43)}
    for sv in (a, b):
        sv.step([(1, prompts[1]), (2, prompts[2])])
    g = a.m.capture_decode(3, 8)
    for sv in (a, b):
        sv.step([(3, prompts[3])])
    nxt = {r: toks(12, cfg["vocab"], 50 + r) for r in prompts}
    for i in range(12):
        parts = [(r, [nxt[r][i]]) for r in (1, 2, 3)]
        want = torch.cat(b.step(parts))
        entries = []
        for r, tk in parts:
            assert a.cache.reserve(r, a.len[r] + 1)
            entries.append(a.cache.entry(r, tk, a.len[r]))
            a.len[r] += 1
        got = g.replay(entries).double().cpu()
        assert rel(got, want) < bar, f"replay {i}"
        torch.cuda.synchronize()


@pytest.mark.gpu
def test_checkpoint_folder_through_registry_command_line_and_trace_replay(dev, tmp_path, monkeypatch, capsys):
    """config.json + model.safetensors on disk -> registry -> `trace` (steps from standard input, logits to files, pages and slots given back and reused) and `generate`
    (scheduler, engine, sampler) -- both against the restatement"""
    from safetensors.torch import save_file
    from mistralrs_amd import cli, registry, trace
    cfg = config([lru(), par2(), par(mlp=None), lru(mlp=None)], loop=(1, 3, 2))
    w = weights(cfg, 12)
    folder = tmp_path / "model"
    folder.mkdir()
    (folder / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in w.items()}, str(folder / "model.safetensors"))
    assert registry.architecture_of(str(folder)) == "Zumuzen"
    wd = f64(w)
    reqs = {"a": toks(45, cfg["vocab"], 61), "b": toks(20, cfg["vocab"], 62), "c": toks(33, cfg["vocab"], 63)}
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": reqs["a"][:30], "want": [0, 29]}, {"id": "b", "tokens": reqs["b"][:19], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": reqs["a"][30:31], "want": [0]}, {"id": "b", "tokens": reqs["b"][19:], "want": [0]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "c", "tokens": reqs["c"][:2], "want": [1]}, {"id": "a", "tokens": reqs["a"][31:], "want": [13]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "c", "tokens": reqs["c"][2:], "want": [0, 30]}], "end": ["c"]}]
    out = tmp_path / "out"
    monkeypatch.setattr("sys.stdin", io.StringIO("\n".join(json.dumps(s) for s in steps) + "\n"))
    assert trace.main(["--model", str(folder), "--dtype", "float32", "--out", str(out), "--max-tokens", "128", "--state-slots", "2"]) == 0
    printed = capsys.readouterr().out.split("\n")
    assert [l for l in printed if l.startswith("done")] == [f"done {i}" for i in range(4)]
    full = {r: logits_of(cfg, wd, t) for r, t in reqs.items()}
    want = {0: [full["a"][0], full["a"][29]], 1: [full["a"][30], full["b"][19]], 2: [full["c"][1], full["a"][44]], 3: [full["c"][2], full["c"][32]]}
    for n, rows in want.items():
        got = torch.from_numpy(np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(len(rows), cfg["vocab"]).astype(np.float64))
        assert rel(got, torch.stack(rows)) < 5e-5, f"step {n}"
    if not os.path.exists(_lib.path("core")):
        pytest.skip("the sampler's library is not built")
    prompts = [toks(12, cfg["vocab"], 71), toks(3, cfg["vocab"], 72)]
    args = ["generate", "--model", str(folder), "--dtype", "float32", "--max-new-tokens", "4", "--max-tokens", "256", "--max-seqs", "2"]
    for p in prompts:
        args += ["--prompt-ids", ",".join(map(str, p))]
    assert cli.main(args) == 0
    lines = [json.loads(l) for l in capsys.readouterr().out.split("\n") if l.startswith("{")]
    assert len(lines) == 2
    for p, line in zip(prompts, lines):
        ref = list(p)
        for _ in range(4):
            lg = logits_of(cfg, wd, ref)[-1]
            t2 = torch.topk(lg, 2).values
            if float(t2[0] - t2[1]) < 1e-3:
                break
            ref.append(int(lg.argmax()))
        assert line["error"] is None and line["tokens"][:len(ref) - len(p)] == ref[len(p):]
