"""Kebisun decoders (mistralrs_amd.hybrid: norms that join the stream, GlaMixer, LatentAttention with query latent / rotated key part / window / sink / gate, UngatedMoe with the softmax
over all experts, GELU-GLU; csrc/hyb_linattn.hip, csrc/hyb_latent.hip and the options added to csrc/hyb_kernels.hip / hyb_gemm.hip) against the plain float64 restatement in
tests/kebisun_oracle.py.

Every test builds its own small configuration with random bf16-representable weights.  The sharp comparisons run in the all-f32 mode (a wrong key, a lost state, a sink left
out is an O(1) error there, rounding is 1e-6); the bf16 mode (whose latent attention runs on the matrix cores) is held to a rounding-sized bar, its kernels alone to the
rounding of their result.  CPU tests cover what needs no device.
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
from tests import kebisun_oracle as O

D64 = torch.float64


# ---------------------------------------------------------------------------------------------------------------- configurations and weights
def dense(ff=56):
    return {"kind": "dense", "ff": ff}


def moe(experts=6, top=2, ff=24):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}


def _ff(mlp):
    return moe() if mlp == "moe" else dense() if mlp == "dense" else mlp


def gla(heads=4, dim=16, vdim=8, tau=4.0, mlp="moe"):
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}, "mlp": _ff(mlp)}


def lat(heads=4, dim=16, rot_dim=8, vdim=24, kv_rank=48, q_rank=20, size=21, base=500.0, scaling=(4.0, 8.0, 1.0, 64), scale=None, mlp="dense"):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank, "scale": scale if scale is not None else (dim + rot_dim) ** -0.5,
         "rot": {"dims": rot_dim, "base": base}}
    if size:
        m["mask"] = {"size": size}
    if scaling:
        m["rot"]["scaling"] = dict(zip(("factor", "fast", "slow", "original"), scaling))
    return {"type": "latent_attention", "mixer": m, "mlp": _ff(mlp)}


def config(layers, vocab=96, width=40, eps=1e-5, scale=3.0):
    return {"architecture": "Kebisun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale}, "layers": layers}


def weights(cfg, seed=0, rank=5, slow=False):
    """slow: decays close to one, so that a state written early is still read hundreds of tokens later"""
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]
    w = {}

    def rnd(*shape, scale=1.0, shift=0.0):
        return (torch.randn(*shape, generator=g) * scale + shift).to(torch.bfloat16)
    a = W ** -0.5 / max(cfg["embedding"]["scale"], 1.0)      # sublayers read the stream itself: undo its size
    w["embed"], w["head"], w["final.norm"] = rnd(cfg["vocab"], W), rnd(cfg["vocab"], W, scale=W ** -0.5), rnd(W, scale=0.2, shift=1.0)
    for i, L in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", L["mixer"], L.get("mlp")
        for n in ("1", "2") if f else ("1",):
            w[p + "norm" + n], w[p + "ls" + n] = rnd(W, scale=0.2, shift=1.0), rnd(W, scale=0.3, shift=1.0)
        q = p + "mix."
        H, D, Dv = m["heads"], m["dim"], m["vdim"]
        w[q + "o"] = rnd(W, H * Dv, scale=(H * Dv) ** -0.5)
        if L["type"] == "gla":
            w[q + "q"], w[q + "k"], w[q + "v"], w[q + "g"] = rnd(H * D, W, scale=2 * a), rnd(H * D, W, scale=2 * a), rnd(H * Dv, W, scale=2 * a), rnd(H * Dv, W, scale=3 * a)
            w[q + "a1"], w[q + "a2"], w[q + "a2.b"] = rnd(rank, W, scale=2 * a), rnd(H * D, rank, scale=rank ** -0.5), rnd(H * D, scale=0.5, shift=5.0 if slow else 0.5)
            w[q + "norm"] = rnd(Dv, scale=0.2, shift=1.0)
        else:
            R, Dr, Q = m["kv_rank"], m["rot_dim"], m["q_rank"]
            w[q + "dq"], w[q + "dq.norm"], w[q + "uq"] = rnd(Q, W, scale=2 * a), rnd(Q, scale=0.2, shift=1.2), rnd(H * (D + Dr), Q, scale=1.5 * Q ** -0.5)
            w[q + "dkv"], w[q + "dkv.norm"] = rnd(R + Dr, W, scale=2 * a), rnd(R, scale=0.2, shift=1.2)
            w[q + "uk"], w[q + "uv"] = rnd(H * D, R, scale=1.5 * R ** -0.5), rnd(H * Dv, R, scale=R ** -0.5)
            w[q + "sink"], w[q + "g"] = rnd(H, scale=1.0, shift=0.5), rnd(H * Dv, W, scale=3 * a)
        if f and f["kind"] == "dense":
            w[p + "mlp.gate"], w[p + "mlp.up"], w[p + "mlp.down"] = rnd(f["ff"], W, scale=2 * a), rnd(f["ff"], W, scale=2 * a), rnd(W, f["ff"], scale=f["ff"] ** -0.5)
        elif f:
            E, ff = f["router"]["experts"], f["expert"]["ff"]
            w[p + "mlp.router"] = rnd(E, W, scale=4 * a)
            for e in range(E):
                w[f"{p}mlp.e{e}.up"], w[f"{p}mlp.e{e}.down"] = rnd(ff, W, scale=2 * a), rnd(W, ff, scale=ff ** -0.5)
    return w


def f64(w):
    return {k: v.to(D64) for k, v in w.items()}


STACK = [lat(), gla(), lat(heads=3, dim=8, rot_dim=16, vdim=32, kv_rank=32, q_rank=24, size=9, mlp="moe"), gla(heads=2, dim=24, vdim=40, tau=1.0, mlp=None), lat(scaling=None, size=70, mlp=None),
         gla(heads=3, dim=8, vdim=12, tau=9.5, mlp="dense")]


class Served:
    """A model on the device with its caches, stepped the way the engine and the trace runner step it."""

    def __init__(self, cfg, w, dev, dtype="float32", max_tokens=512, slots=4, block_size=32):
        from mistralrs_amd.hybrid import SPEC_READERS, HybridCache, HybridDecoder
        self.bs = block_size
        self.m = HybridDecoder(SPEC_READERS[cfg["architecture"]](cfg), dev, dtype, num_blocks=-(-max_tokens // block_size) + slots + 1, block_size=block_size, state_slots=slots)
        self.m.load_weights(w.__getitem__)
        self.cache = HybridCache(self.m)
        self.len = {}

    def step(self, parts):
        """parts: [(request id, tokens)]; logits of every row, split per part"""
        from mistralrs_amd.hybrid import RaggedBatch
        entries = []
        for rid, tk in parts:
            p0 = self.len.get(rid, 0)
            assert self.cache.reserve(rid, p0 + len(tk)), "out of pages / slots"
            entries.append(self.cache.entry(rid, tk, p0, range(len(tk))))
            self.len[rid] = p0 + len(tk)
        out = self.m.forward_batch(RaggedBatch.build(entries, self.bs, self.m.device)).double().cpu()
        res, r = [], 0
        for _, tk in parts:
            res.append(out[r:r + len(tk)])
            r += len(tk)
        return res

    def end(self, rid):
        self.cache.release(rid)
        self.len.pop(rid, None)


def rel(a, b):
    return float((a - b).norm() / (b.norm() + 1e-30))


def close(a, b, bar):
    """f32 mode (bar < 1e-3): the whole tensor within `bar`.  bf16 mode: the typical row within `bar`, at most one row in ten above five times that."""
    if bar < 1e-3:
        return rel(a, b) < bar
    rows = (a - b).reshape(-1, a.shape[-1]).norm(dim=1) / (b.reshape(-1, b.shape[-1]).norm(dim=1) + 1e-30)
    return float(rows.median()) < bar and float((rows > 5 * bar).double().mean()) <= 0.1


def toks(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def logits_of(cfg, wd, t):
    return O.forward(cfg, wd, t)[0]


def _batch(dev, parts, bs=32, blocks=None):
    """a RaggedBatch of [(first position, rows, state slot)] over made-up block tables"""
    from mistralrs_amd.hybrid import RaggedBatch
    entries, nb = [], 0
    for k, (p0, n, slot) in enumerate(parts):
        need = -(-(p0 + n) // bs)
        blk = blocks[k] if blocks else list(range(nb + 1, nb + 1 + need))
        nb += need
        entries.append({"tokens": [0] * n, "pos0": p0, "slot": slot, "blocks": blk, "want": []})
    return RaggedBatch.build(entries, bs, dev)


# ---------------------------------------------------------------------------------------------------------------- no device needed
def test_config_reader_takes_every_size_and_constant_from_the_file():
    from mistralrs_amd.hybrid import GlaSpec, GluSpec, LatentAttentionSpec, UngatedMoeSpec, kebisun_spec
    cfg = config([lat(heads=5, dim=10, rot_dim=6, vdim=14, kv_rank=22, q_rank=18, size=17, base=77.0, scaling=(3.0, 9.0, 2.0, 100), scale=0.3, mlp=moe(9, 3, 21)),
                  gla(heads=3, dim=6, vdim=7, tau=3.5, mlp=dense(77)), gla(mlp=None), lat(size=0, scaling=None)], vocab=123, width=56, eps=3e-4, scale=7.5)
    sp = kebisun_spec(cfg)
    assert (sp.vocab, sp.width, sp.eps, sp.norm, sp.join_norms, sp.layer_scale, sp.embed_scale, sp.head, sp.post_norms, sp.streams) == (123, 56, 3e-4, "layer_plain", True, True, 7.5, "head", False, 0)
    a, b, c, d = sp.layers
    assert [l.kind for l in sp.layers] == ["latent_attention", "gla", "gla", "latent_attention"] and [l.prefix for l in sp.layers] == ["l0.", "l1.", "l2.", "l3."]
    m = a.mixer
    assert isinstance(m, LatentAttentionSpec)
    assert (m.heads, m.dim, m.vdim, m.kv_rank, m.scale, m.q_rank, m.rot_dim, m.window, m.sink, m.gate) == (5, 10, 14, 22, 0.3, 18, 6, 17, True, True)
    assert (m.rotary.dims, m.rotary.base, m.rotary.layout) == (6, 77.0, "half") and m.rotary.trig_mult == pytest.approx(0.1 * math.log(3.0) + 1.0, abs=1e-12)
    assert isinstance(a.ff, UngatedMoeSpec) and (a.ff.experts, a.ff.top, a.ff.ff, a.ff.act, a.ff.routing) == (9, 3, 21, "gelu", "all")
    assert isinstance(b.mixer, GlaSpec) and (b.mixer.heads, b.mixer.dim, b.mixer.vdim, b.mixer.tau) == (3, 6, 7, 3.5)
    assert isinstance(b.ff, GluSpec) and (b.ff.ff, b.ff.act) == (77, "gelu_tanh") and c.ff is None
    assert d.mixer.window == 0 and d.mixer.rotary.scaling is None and d.mixer.rotary.trig_mult == 1.0
    for bad in ([{"type": "mamba2", "mixer": {}, "mlp": None}], [gla(mlp={"kind": "glu"})], [lat(rot_dim=5)]):
        with pytest.raises(ValueError):
            kebisun_spec(config(bad))


@pytest.mark.parametrize("dims,base,scaling", [(8, 500.0, (4.0, 8.0, 1.0, 64)), (64, 10000.0, (5.0, 32.0, 1.0, 4096)), (2, 100.0, (8.0, 2.0, 1.0, 10)), (32, 50.0, (16.0, 1000.0, 0.01, 7)),
                                               (16, 10000.0, (1.0, 4.0, 4.0, 512))])
def test_ramped_rotary_frequencies(dims, base, scaling):
    from mistralrs_amd.hybrid import RotarySpec
    sc = dict(zip(("factor", "fast", "slow", "original"), scaling))
    f, mult = O.yarn({"dims": dims, "base": base, "scaling": sc})
    r = RotarySpec(dims, base, sc, "half")
    assert np.allclose(r.frequencies(), np.array(f, dtype=np.float64), rtol=1e-6, atol=0) and r.trig_mult == pytest.approx(mult)
    assert np.allclose(RotarySpec(dims, base, None, "half").frequencies(), [base ** (-2.0 * i / dims) for i in range(dims // 2)], rtol=1e-6)


def test_registry_and_synthetic_weights_know_the_architecture():
    from mistralrs_amd import registry
    from mistralrs_amd.hybrid import FEED_FORWARDS, MIXERS, SPEC_READERS, kebisun_spec, synthetic_weights
    assert "Kebisun" in registry.ARCHITECTURES and "Kebisun" in SPEC_READERS and {"gla", "latent_attention"} <= set(MIXERS) and "moe_ungated" in FEED_FORWARDS
    cfg = config(STACK)
    get = synthetic_weights(kebisun_spec(cfg), "cpu", 1)
    for name, t in weights(cfg).items():
        if name.endswith((".a1", ".a2")):
            assert get(name).shape[name.endswith("2") ^ 1] == t.shape[name.endswith("2") ^ 1], name   # the inner size is the generator's choice
        else:
            assert tuple(get(name).shape) == tuple(t.shape), name
    for name in ("l0.norm1.b", "l3.norm2", "l3.ls2", "l1.mlp.router.b"):
        with pytest.raises(KeyError):
            get(name)


def test_batch_knows_its_context_blocks_and_visible_pairs():
    """blocks wholly before a window are left out of the gathered context, an entry's blocks stay consecutive; the pair count equals a count by hand"""
    b = _batch("cpu", [(70, 5, 0), (0, 3, 0), (31, 2, 0)], bs=8, blocks=[[11, 12, 13, 14, 15, 16, 17, 18, 19, 20], [3], [5, 6, 7, 8, 9]])
    tables, src, n = b.context_blocks(20, 8)           # first rows see from 51, 0, 12 on: blocks 6, 0, 1
    assert src.tolist() == [17, 18, 19, 20, 3, 6, 7, 8, 9] and n == 9
    assert tables[0, 6:10].tolist() == [0, 1, 2, 3] and tables[1, 0].item() == 4 and tables[2, 1:5].tolist() == [5, 6, 7, 8]
    tables, src, n = b.context_blocks(0, 8)
    assert n == 16 and src.tolist()[:10] == list(range(11, 21))
    for win in (0, 1, 4, 20, 33, 71, 1000):
        pairs = sum(min(p0 + i + 1, win) if win else p0 + i + 1 for p0, m in ((70, 5), (0, 3), (31, 2)) for i in range(m))
        assert b.visible_pairs(win)[0] == pairs, win


def test_restatement_pieces():
    """the oracle's own building blocks on hand-computed values"""
    # one head, two key channels that decay differently: what is written along channel 0 fades by 1 / 2 per row, channel 1 keeps
    k = torch.tensor([[1.0, 0.0], [0.0, 1.0], [0.0, 0.0]], dtype=D64).view(3, 1, 2)
    v = torch.tensor([[2.0, 3.0], [5.0, 7.0], [9.0, 9.0]], dtype=D64).view(3, 1, 2)
    q = torch.tensor([[1.0, 1.0], [1.0, 0.0], [1.0, 1.0]], dtype=D64).view(3, 1, 2)
    al = torch.tensor([0.5, 1.0], dtype=D64).expand(3, 1, 2)
    o, S = O.gla_cell(q, k, v, al, torch.zeros(1, 2, 2, dtype=D64))
    assert o.view(3, 2).tolist() == [[2.0, 3.0], [1.0, 1.5], [5.5, 7.75]] and S[0].tolist() == [[0.5, 0.75], [5.0, 7.0]]
    w = {"a1": torch.eye(2, dtype=D64), "a2": torch.eye(2, dtype=D64), "a2.b": torch.tensor([0.0, 1.0], dtype=D64)}
    al = O.gla_decay(torch.tensor([[0.0, -1.0]], dtype=D64), w, "", {"heads": 1, "dim": 2, "tau": 2.0})
    assert torch.allclose(al.view(2), torch.tensor([0.5 ** 0.5, 0.5 ** 0.5], dtype=D64))
    # the sink takes weight and gives nothing
    p = O.softmax_sink(torch.tensor([0.0, math.log(3.0)], dtype=D64), torch.tensor(math.log(4.0), dtype=D64))
    assert torch.allclose(p, torch.tensor([1 / 8, 3 / 8], dtype=D64))
    # rotation: the pair (i, i + dims / 2), values past dims pass; with scaling the fast pairs keep their frequency, the slow ones are divided, cos and sin are stretched
    x = torch.zeros(3, 6, dtype=D64)
    x[:, 1], x[:, 5] = 1.0, 7.0
    r = O.rotate_half(x, torch.arange(3), {"dims": 4, "base": 100.0})
    assert torch.allclose(r[:, 1], torch.cos(torch.arange(3, dtype=D64) * 0.1)) and torch.allclose(r[:, 3], torch.sin(torch.arange(3, dtype=D64) * 0.1)) and r[:, 5].tolist() == [7.0] * 3
    f, mult = O.yarn({"dims": 8, "base": 10000.0, "scaling": {"factor": 4.0, "original": 1024, "fast": 32.0, "slow": 1.0}})
    place = lambda t: 8 * math.log(1024 / (2 * math.pi * t)) / (2 * math.log(10000.0))
    lo, hi = math.floor(place(32.0)), math.ceil(place(1.0))
    assert (lo, hi) == (0, 3) and f[0] == 1.0 and f[3] == pytest.approx(1e-3 / 4) and f[1] == pytest.approx(0.1 / 4 / 3 + 0.1 * 2 / 3) and mult == pytest.approx(1.1386294361)
    # norms, activations, routing
    y = O.layer_norm(torch.tensor([[1.0, 3.0]], dtype=D64), torch.tensor([2.0, 5.0], dtype=D64), 0.0)
    assert torch.allclose(y, torch.tensor([[-2.0, 5.0]], dtype=D64))
    z = torch.linspace(-3, 3, 7, dtype=D64)
    assert torch.allclose(O.gelu_erf(z), torch.nn.functional.gelu(z)) and torch.allclose(O.gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh"))
    ids, wts = O.route(torch.tensor([[2.0, 2.0, 0.5, -1.0]], dtype=D64), {"router": torch.eye(4, dtype=D64)}, "", {"router": {"top": 2}})
    assert ids.tolist() == [[0, 1]] and torch.allclose(wts, torch.softmax(torch.tensor([[2.0, 2.0, 0.5, -1.0]], dtype=D64), -1)[:, :2])


def test_restatement_decodes_token_by_token_like_whole_prompts():
    """the oracle carries states between calls: whole prompt == portions == single tokens"""
    cfg = config(STACK)
    wd = f64(weights(cfg, 3))
    t = toks(60, cfg["vocab"], 4)
    want, after, _ = O.forward(cfg, wd, t)
    got, st, at = [], None, 0
    for n in (1, 2, 20, 1, 36):
        lg, _, st = O.forward(cfg, wd, t[at:at + n], st, at)
        got.append(lg)
        at += n
    assert rel(torch.cat(got), want) < 1e-12 and after.shape == (len(STACK), 60, cfg["width"])


# ---------------------------------------------------------------------------------------------------------------- kernels alone (GPU)
@pytest.mark.gpu
@pytest.mark.parametrize("W", [40, 257, 1028])
def test_norm_into_the_stream(dev, W):
    """x += norm(y) w from a product and from routed outputs; the rounded copy is the updated row; one launch each"""
    from mistralrs_amd.hybrid import _call
    _lib.load("hybrid")
    g = torch.Generator().manual_seed(W)
    T, top = 5, 3
    y, x, w, b = torch.randn(T, W, generator=g) * 3 + 1, torch.randn(T, W, generator=g), torch.randn(W, generator=g), torch.randn(W, generator=g)
    d, wts = torch.randn(T * top, W, generator=g), torch.rand(T * top, generator=g)
    place = torch.randperm(T * top, generator=g).to(torch.int32)
    summed = (wts.view(T, top, 1).double() * d.double()[place.long()].view(T, top, W)).sum(1)
    for dt, TT in ((2, torch.float32), (1, torch.bfloat16)):
        for routed in (False, True):
            for bias in (None, b):
                xd, out = x.to(dev), torch.empty(T, W, dtype=TT, device=dev)
                _call("mrs_hyb_layernorm_join", None if routed else y.to(dev), W, d.to(dev) if routed else None, place.to(dev) if routed else None, wts.to(dev) if routed else None, top,
                      w.to(dev), bias.to(dev) if bias is not None else None, xd, W, out, T, W, 1e-5, dt)
                want = x.double() + O.layer_norm(summed if routed else y.double(), w.double(), 1e-5) + (0 if bias is None else b.double())
                assert rel(xd.double().cpu(), want) < 1e-6
                assert torch.equal(out.cpu(), xd.cpu().to(TT))


@pytest.mark.gpu
def test_scaled_embedding_rows(dev):
    from mistralrs_amd.hybrid import _call
    _lib.load("hybrid")
    g = torch.Generator().manual_seed(1)
    table = torch.randn(30, 50, generator=g).to(torch.bfloat16)
    ids = torch.tensor([3, 29, 0, 3], dtype=torch.int32)
    x, h = torch.empty(4, 50, device=dev), torch.empty(4, 50, dtype=torch.bfloat16, device=dev)
    _call("mrs_hyb_embed_scaled", ids.to(dev), table.to(dev), x, h, 4, 50, 30, 2.7, 1)
    want = table[ids.long()].float() * 2.7
    assert torch.equal(x.cpu(), want) and torch.equal(h.cpu(), want.to(torch.bfloat16))


@pytest.mark.gpu
@pytest.mark.parametrize("qr,R,rot,dims", [(20, 48, 8, 8), (0, 7, 6, 4), (33, 129, 2, 2), (5, 16, 0, 0), (300, 512, 64, 64)])
def test_latent_row_and_query_latent(dev, qr, R, rot, dims):
    """the query latent and the latent are normed by their own root mean squares, the key part is rotated and not normed; all end up in the right place of the right page"""
    from mistralrs_amd.hybrid import _call
    _lib.load("hybrid")
    g = torch.Generator().manual_seed(R)
    T, bs = 6, 4
    ld = qr + R + rot + 3
    u, qw, cw = torch.randn(T, ld, generator=g), torch.randn(max(qr, 1), generator=g), torch.randn(R, generator=g)
    pos = torch.tensor([0, 1, 5, 700, 2, 3], dtype=torch.int32)
    slots = torch.tensor([4, 5, 9, 0, 14, 15], dtype=torch.int64)
    rcfg = {"dims": dims, "base": 50.0, "scaling": {"factor": 4.0, "fast": 2.0, "slow": 0.5, "original": 100}} if dims else None
    f, mult = O.yarn(rcfg) if dims else ([0.0], 1.0)
    cq, cache = torch.empty(T, max(qr, 1), device=dev), torch.zeros(4, bs, R + rot, device=dev)
    _call("mrs_hyb_latent_prep", u.to(dev), ld, qr, R, rot, dims, qw.to(dev) if qr else None, cw.to(dev), torch.tensor(f).float().to(dev), mult, pos.to(dev), slots.to(dev),
          cq if qr else None, cache, 1e-5, T, 2)
    ud = u.double()
    if qr:
        assert rel(cq.double().cpu(), O.rms_norm(ud[:, :qr], qw.double(), 1e-5)) < 2e-6
    c = O.rms_norm(ud[:, qr:qr + R], cw.double(), 1e-5)
    k = O.rotate_half(ud[:, qr + R:qr + R + rot], pos, rcfg)
    for t in range(T):
        row = cache[int(slots[t]) // bs, int(slots[t]) % bs].double().cpu()
        assert rel(row[:R], c[t]) < 2e-6 and (not rot or rel(row[R:], k[t]) < 5e-5), t
    used = set(slots.tolist())
    assert all(float(cache.view(-1, R + rot)[s].abs().max()) == 0.0 for s in range(16) if s not in used)


@pytest.mark.gpu
@pytest.mark.parametrize("H,D,rot,dims", [(4, 16, 8, 8), (3, 5, 6, 4), (1, 64, 64, 64), (2, 7, 0, 0)])
def test_latent_queries_rotate_behind_the_plain_part_or_in_the_tail_of_the_absorbed_query(dev, H, D, rot, dims):
    from mistralrs_amd.hybrid import _call
    _lib.load("hybrid")
    g = torch.Generator().manual_seed(D)
    T, R = 4, 9
    qf = torch.randn(T, H * (D + rot) + 2, generator=g)
    pos = torch.tensor([0, 3, 250, 9], dtype=torch.int32)
    rcfg = {"dims": dims, "base": 300.0} if dims else None
    f = torch.tensor(O.yarn(rcfg)[0] if dims else [0.0]).float().to(dev)
    q, qa = torch.empty(T, H * (D + rot), device=dev), torch.zeros(T, H * (R + rot), device=dev)
    view = qf[:, :H * (D + rot)].double().view(T, H, D + rot)
    turned = O.rotate_half(view[..., D:], pos, rcfg)
    _call("mrs_hyb_latent_query", qf.to(dev), qf.shape[1], H, D, R, rot, dims, f, 1.0, pos.to(dev), q, None, T, 2)
    assert rel(q.double().cpu().view(T, H, -1), torch.cat([view[..., :D], turned], -1)) < 3e-5
    q.zero_()
    _call("mrs_hyb_latent_query", qf.to(dev), qf.shape[1], H, D, R, rot, dims, f, 1.0, pos.to(dev), q, qa, T, 2)
    assert torch.equal(q.cpu().view(T, H, -1)[..., :D].double(), view[..., :D])
    got = qa.double().cpu().view(T, H, R + rot)
    assert float(got[..., :R].abs().max()) == 0.0 and (not rot or rel(got[..., R:], turned) < 3e-5)


@pytest.mark.gpu
def test_context_rows_and_key_parts_of_whole_blocks(dev):
    from mistralrs_amd.hybrid import _call
    _lib.load("hybrid")
    g = torch.Generator().manual_seed(2)
    bs, R, rot, H, D = 4, 6, 3, 2, 5
    cache = torch.randn(7, bs, R + rot, generator=g).to(torch.bfloat16)
    src = torch.tensor([5, 2, 3], dtype=torch.int32)
    c, k = torch.zeros(12, R, dtype=torch.bfloat16, device=dev), torch.zeros(12, H * (D + rot), dtype=torch.bfloat16, device=dev)
    _call("mrs_hyb_latent_context", cache.to(dev), src.to(dev), c, k, 3, bs, R, rot, H, D, 1)
    rows = cache[src.long()].view(12, R + rot)
    assert torch.equal(c.cpu(), rows[:, :R])
    kv = k.cpu().view(12, H, D + rot)
    assert torch.equal(kv[..., D:], rows[:, None, R:].expand(12, H, rot)) and float(kv[..., :D].abs().max()) == 0.0


@pytest.mark.gpu
@pytest.mark.parametrize("n", [1, 33, 256])
def test_activations_and_gates(dev, n):
    from mistralrs_amd.hybrid import _call
    _lib.load("hybrid")
    g = torch.Generator().manual_seed(n)
    gu, gate = torch.randn(6, 2 * n, generator=g) * 3, torch.randn(6, n + 4, generator=g) * 3
    u = gu.to(dev)
    for dt, TT, bar in ((2, torch.float32, 1e-6), (1, torch.bfloat16, 4e-3)):
        o = torch.empty(6, n, dtype=TT, device=dev)
        _call("mrs_hyb_glu_gelu", u, o, 6, n, dt)
        assert rel(o.double().cpu(), O.gelu_tanh(gu[:, :n].double()) * gu[:, n:].double()) < bar
        flat = u[:, :n].contiguous()
        _call("mrs_hyb_gelu_erf", flat, o, 6, n, dt)
        assert rel(o.double().cpu(), O.gelu_erf(gu[:, :n].double())) < bar
        _call("mrs_hyb_sigmoid_gate", flat, gate.to(dev), n + 4, o, 6, n, dt)
        assert rel(o.double().cpu(), gu[:, :n].double() * torch.sigmoid(gate[:, :n].double())) < bar


@pytest.mark.gpu
@pytest.mark.parametrize("M,N,K", [(1, 24, 40), (2, 7, 33), (4, 65, 512), (8, 5, 1000)])
@pytest.mark.parametrize("ep", [1, 2, 3, 4])
def test_row_products_that_write_activated_operands(dev, M, N, K, ep):
    from mistralrs_amd.hybrid import _call
    _lib.load("hybrid")
    g = torch.Generator().manual_seed(N + ep)
    glu = ep > 2
    a, w = torch.randn(M, K, generator=g).to(torch.bfloat16), (torch.randn(2 * N if glu else N, K, generator=g) * 2 * K ** -0.5).to(torch.bfloat16)
    z = a.double() @ w.double().T
    want = {1: lambda: torch.clamp(z, min=0) ** 2, 2: lambda: O.gelu_erf(z), 3: lambda: O.silu(z[:, :N]) * z[:, N:], 4: lambda: O.gelu_tanh(z[:, :N]) * z[:, N:]}[ep]()
    for dt, TT, bar in ((2, torch.float32, 2e-6), (1, torch.bfloat16, 4e-3)):
        o = torch.empty(M, N, dtype=TT, device=dev)
        _call("mrs_hyb_gemv_ep", a.to(dev, TT), w.to(dev, TT), o, M, N, K, K, K, N, dt, None, 0, 0, None, 1, ep)
        assert rel(o.double().cpu(), want) < bar
    if not glu:   # a weight per row, the rows gathered from f32 source rows
        E, R = 3, 11
        ws = (torch.randn(E, N, K, generator=g) * 2 * K ** -0.5).to(torch.bfloat16)
        src = torch.randn(M, K, generator=g)
        grp, route = torch.randint(0, E, (R,), generator=g).to(torch.int32), torch.randint(0, 2 * M, (R,), generator=g).to(torch.int32)
        rows = src[(route // 2).long()].double()
        zz = torch.stack([ws[grp[r].long()].double() @ rows[r] for r in range(R)])
        o = torch.empty(R, N, device=dev)
        _call("mrs_hyb_gemv_ep", src.to(dev), ws.float().to(dev), o, R, N, K, K, K, N, 2, grp.to(dev), N * K, 2, route.to(dev), 2, ep)
        assert rel(o.double().cpu(), torch.clamp(zz, min=0) ** 2 if ep == 1 else O.gelu_erf(zz)) < 2e-6


@pytest.mark.gpu
@pytest.mark.parametrize("E,top,W", [(6, 2, 40), (16, 4, 64), (70, 7, 33), (3, 3, 8), (5, 1, 12)])
def test_router_scores_over_all_experts(dev, E, top, W):
    from mistralrs_amd.hybrid import _call
    _lib.load("hybrid")
    g = torch.Generator().manual_seed(E)
    h, wr = torch.randn(11, W, generator=g), torch.randn(E, W, generator=g)
    h[3] = 0.0              # all scores equal: the lower indices
    ids, wts = torch.empty(11 * top, dtype=torch.int32, device=dev), torch.empty(11 * top, device=dev)
    _call("mrs_hyb_route_softmax_topk", h.to(dev), wr.to(dev), 11, W, E, top, 1.0, ids, wts)
    want_ids, want_w = O.route(h.double(), {"router": wr.double()}, "", {"router": {"top": top}})
    assert torch.equal(ids.cpu().view(11, top).long(), want_ids) and rel(wts.double().cpu().view(11, top), want_w) < 2e-6


# ---- gated linear attention
def _gla_rows(T, H, D, Dv, seed, slow=False):
    g = torch.Generator().manual_seed(seed)
    q, k, v = torch.randn(T, H, D, generator=g), torch.randn(T, H, D, generator=g), torch.randn(T, H, Dv, generator=g)
    z = torch.randn(T, H, D, generator=g) * 2 + (6.0 if slow else 0.0)
    return q, k, v, z


@pytest.mark.gpu
@pytest.mark.parametrize("seg", [0, 32, 64], ids=["chains", "segments_of_32", "segments_of_64"])
@pytest.mark.parametrize("H,D,Dv,tau", [(4, 16, 8, 4.0), (2, 32, 32, 16.0), (2, 64, 16, 1.0), (3, 7, 5, 2.0), (1, 130, 3, 16.0), (2, 128, 260, 16.0), (1, 300, 70, 8.0), (5, 1, 1, 3.0), (1, 48, 130, 0.5)])
def test_recurrence_over_portions_single_rows_and_reused_slots(dev, H, D, Dv, tau, seg):
    """three sequences through slots that hold a former owner's numbers: portions of several sizes (some longer than two segments) beside single rows, every entry as one chain
    or its segments side by side, every row against the restatement on the whole sequence; single-row steps through the one-launch form as well"""
    from mistralrs_amd.hybrid import _call
    _lib.load("hybrid")
    lens = (250, 151, 9)
    qm = float(np.float32(D) ** np.float32(-0.5))
    seqs = [_gla_rows(n, H, D, Dv, 10 * D + k, slow=k == 0) for k, n in enumerate(lens)]   # the longest one decays slowly: what a segment is handed matters
    zb = torch.randn(H * D, generator=torch.Generator().manual_seed(7))
    want = []
    for q, k, v, z in seqs:
        al = torch.sigmoid(z.double() + zb.double().view(H, D)) ** (1.0 / tau)
        want.append(O.gla_cell(q.double() * D ** -0.5, k.double(), v.double(), al, torch.zeros(H, D, Dv, dtype=D64))[0].reshape(-1, H * Dv))
    nv, nk, pad = H * Dv, H * D, 3
    ld = nv + 2 * nk + pad
    state = torch.full((5, H, D, Dv), 1e6, device=dev)
    state[1] = float("nan")
    got, at = [[] for _ in seqs], [0, 0, 0]

    def run(ns, slots=(3, 0, 4)):
        parts = [(j, n) for j, n in enumerate(ns) if n]
        b = _batch(dev, [(at[j], n, slots[j]) for j, n in parts])
        rows = []
        for j, n in parts:
            q, k, v, _ = seqs[j]
            s = slice(at[j], at[j] + n)
            rows.append(torch.cat([v[s].reshape(n, -1), torch.zeros(n, pad), k[s].reshape(n, -1), q[s].reshape(n, -1)], 1))
        u = torch.cat(rows).to(dev)
        z = torch.cat([seqs[j][3][at[j]:at[j] + n].reshape(n, -1) for j, n in parts]).to(dev)
        T = u.shape[0]
        _call("mrs_hyb_gla_decays", z, zb.to(dev), T, nk, 1.0 / tau)
        y = torch.empty(T, nv, device=dev)
        table, nseg, carry, dec = b.entry_table(), len(parts), None, None
        if seg:
            *table, nseg = b.segment_table(seg)
            carry, dec = torch.empty(nseg, H, D, Dv, device=dev), torch.empty(nseg, H, D, device=dev)
        _call("mrs_hyb_gla_scan", u, ld, nv + pad, nv + pad + nk, z, state, y, b.seq_pos0, b.seq_slot, *table, carry, dec, T, len(parts), nseg, H, D, Dv, qm)
        r = 0
        for j, n in parts:
            got[j].append(y[r:r + n].double().cpu())
            r += n
            at[j] += n
    run([30, 2, 0])
    run([1, 1, 1])
    run([2, 5, 3])
    run([1, 0, 2])
    run([150, 64, 3])
    run([66, 79, 0])
    assert at == list(lens)
    for j in range(3):
        assert rel(torch.cat(got[j]), want[j]) < 2e-5, j
    assert bool((state[2] == 1e6).all()) and bool(torch.isnan(state[1]).all())


@pytest.mark.gpu
@pytest.mark.parametrize("dt", [2, 1], ids=["f32", "bf16"])
@pytest.mark.parametrize("H,D,Dv,rank,tau", [(4, 16, 8, 5, 4.0), (2, 64, 128, 16, 16.0), (3, 7, 5, 1, 1.0), (1, 256, 512, 40, 8.0), (2, 1, 1, 3, 2.0), (1, 9, 1030, 2, 2.0)])
def test_single_row_step_in_one_launch(dev, H, D, Dv, rank, tau, dt):
    """two rounds of three single rows (one fresh over a NaN-filled slot, two continuing): decays from the projection's first step, state, read-out, head norm and SiLU gate"""
    from mistralrs_amd.hybrid import _call
    _lib.load("hybrid")
    g = torch.Generator().manual_seed(D + Dv)
    TT = torch.float32 if dt == 2 else torch.bfloat16
    nv, nk = H * Dv, H * D
    ld = 2 * nv + 2 * nk + rank + 1
    cols = (nv, nv + nk, nv + 2 * nk, 2 * nv + 2 * nk)
    wa2, zb, nw = torch.randn(nk, rank, generator=g).to(torch.bfloat16), torch.randn(nk, generator=g), torch.randn(Dv, generator=g)
    state = torch.full((4, H, D, Dv), float("nan"), device=dev)
    S = [torch.zeros(H, D, Dv, dtype=D64)] + [torch.randn(H, D, Dv, generator=g).double() for _ in range(2)]
    slots, pos = (2, 0, 3), (0, 9, 40)
    for e in (1, 2):
        state[slots[e]] = S[e].float().to(dev)
    for step in range(2):
        u = torch.randn(3, ld, generator=g)
        b = _batch(dev, [(pos[e] + step, 1, slots[e]) for e in range(3)])
        out = torch.empty(3, nv, dtype=TT, device=dev)
        _call("mrs_hyb_gla_step", u.to(dev), ld, *cols, rank, wa2.to(dev, TT), zb.to(dev), nw.to(dev), state, out, b.seq_start, b.seq_pos0, b.seq_slot, 3, 3, H, D, Dv,
              float(np.float32(D) ** np.float32(-0.5)), 1.0 / tau, 1e-5, dt)
        for e in range(3):
            r = u[e].double()
            a1 = (u[e, cols[3]:cols[3] + rank].to(TT)).double()
            al = (torch.sigmoid(wa2.double() @ a1 + zb.double()) ** (1.0 / tau)).view(1, H, D)
            o, S[e] = O.gla_cell(r[cols[1]:cols[2]].view(1, H, D) * D ** -0.5, r[cols[0]:cols[1]].view(1, H, D), r[:nv].view(1, H, Dv), al, S[e])
            want = (O.rms_norm(o, nw.double(), 1e-5).reshape(nv)) * O.silu(r[cols[2]:cols[3]])
            assert rel(out[e].double().cpu(), want) < (5e-6 if dt == 2 else 5e-3), (step, e)
            assert rel(state[slots[e]].double().cpu(), S[e]) < 5e-6, (step, e)
    assert bool(torch.isnan(state[1]).all())


@pytest.mark.gpu
def test_a_planted_pair_stays_readable_for_hundreds_of_rows_along_its_own_channel(dev):
    """hand-made rows: key e_0 with value u at row 5, all other rows write along e_1 and channel 1 forgets at once; a query e_0 reads decay^distance u hundreds of rows later, over
    portions of 63 / 64 / 65 / 2 / 1 rows, from a slot another sequence left full"""
    from mistralrs_amd.hybrid import _call
    _lib.load("hybrid")
    H, D, Dv, T = 2, 8, 4, 400
    nv, nk = H * Dv, H * D
    ld = nv + 2 * nk
    uval = torch.tensor([1.0, -2.0, 3.0, 0.5], dtype=D64)
    u = torch.zeros(T, ld)
    u[:, nv + nk] = 1.0                    # q of head 0 = e_0
    u[:, nv + 1] = 1.0                     # k of head 0 = e_1
    u[:, :Dv] = 9.0
    u[5, nv + 1], u[5, nv] = 0.0, 1.0
    u[5, :Dv] = uval.float()
    dec = torch.ones(T, nk)
    dec[:, 0], dec[:, 1] = 0.99609375, 0.0
    state = torch.full((3, H, D, Dv), float("nan"), device=dev)
    state[1] = 1e6
    at, outs = 0, []
    for n in (63, 1, 64, 2, 65, 1, 1, 130, 3, 70):
        b = _batch(dev, [(at, n, 1)])
        y = torch.empty(n, nv, device=dev)
        *table, nseg = b.segment_table(32)
        carry, dk = torch.empty(nseg, H, D, Dv, device=dev), torch.empty(nseg, H, D, device=dev)
        _call("mrs_hyb_gla_scan", u[at:at + n].to(dev), ld, nv, nv + nk, dec[at:at + n].to(dev), state, y, b.seq_pos0, b.seq_slot, *table, carry, dk, n, 1, nseg, H, D, Dv, 1.0)
        outs.append(y.double().cpu())
        at += n
    y = torch.cat(outs)[:, :Dv]
    t = torch.arange(T, dtype=D64)
    want = torch.where((t >= 5).view(T, 1), (0.99609375 ** (t - 5)).view(T, 1) * uval, torch.zeros(T, Dv, dtype=D64))
    assert float((y - want).abs().max()) < 1e-5 and float(want[399].abs().max()) > 0.5
    assert torch.isnan(state[0]).all() and torch.isnan(state[2]).all()


# ---- latent attention
class LatentRig:
    """One latent attention module with given sizes over made-up pages: `rows` of every position of some sequences (latent | key part) lie in shuffled pages, unused page slots hold
    NaN.  `run` attends queries of a batch through the expanded form or through the cached rows; `want` restates it in float64 from the same (rounded) numbers."""

    def __init__(self, dev, dtype, H, D, Dr, Dv, R, window, bs=8, scale=0.4, pages=128, seed=0):
        from mistralrs_amd.hybrid import HybridDecoder, HybridSpec, LatentAttentionSpec, LayerSpec
        sp = LatentAttentionSpec(H, D, Dv, R, scale, 4, Dr, None, window, True, True)
        self.m = HybridDecoder(HybridSpec(8, 16, 1e-5, [LayerSpec("latent_attention", sp, None, "l0.")]), dev, dtype, num_blocks=pages, block_size=bs, state_slots=1)
        self.x, self.s, self.bs, self.dev, self.TT = self.m.layers[0].mixer, sp, bs, dev, self.m.torch_dtype
        self.g = torch.Generator().manual_seed(seed)
        q = lambda *s, scale=1.0: (torch.randn(*s, generator=self.g) * scale).to(torch.bfloat16)
        self.uk, self.uv, self.sink = q(H * D, R, scale=R ** -0.5), q(H * Dv, R, scale=R ** -0.5), q(H)
        self.x.w_ukT = self.uk.view(H, D, R).transpose(1, 2).to(dev, self.TT).contiguous()
        self.x.w_uk, self.x.w_uv = self.uk.to(dev, self.TT), self.uv.view(H, Dv, R).to(dev, self.TT)
        self.x.sink = self.sink.float().to(dev)
        self.order = (torch.randperm(pages - 1, generator=self.g) + 1).tolist()
        self.seqs = []

    def add(self, rows):
        """rows [P, R + Dr] (bf16-representable) of a sequence's positions"""
        need = -(-rows.shape[0] // self.bs)
        blk = [self.order.pop() for _ in range(need)]
        if not self.seqs:
            self.x.c_cache.fill_(float("nan"))
        for j in range(rows.shape[0]):
            self.x.c_cache[blk[j // self.bs], 0, j % self.bs] = rows[j].to(self.dev, self.TT)
        self.seqs.append((rows.double(), blk))

    def run(self, q, gate, parts, expanded):
        """parts [(sequence, first position, rows)], q [T, H, D + Dr], gate [T, H * Dv] (nullable)"""
        s, m, x = self.s, self.m, self.x
        b = _batch(self.dev, [(p0, n, 0) for _, p0, n in parts], self.bs, [self.seqs[k][1] for k, _, _ in parts])
        T = q.shape[0]
        qd = q.reshape(T, -1).to(self.dev, self.TT)
        gd = gate.to(self.dev) if gate is not None else None
        out = torch.empty(T, s.heads * s.vdim, dtype=self.TT, device=self.dev)
        if expanded:
            tables, k, v = x.expand_context(b, s.window)
            x.attend_expanded(qd, k, v, tables, b, out, gd, s.heads * s.vdim, s.window)
        else:
            E, R = s.dim + s.rot_dim, s.kv_rank
            qa = torch.zeros(T, s.heads * (R + s.rot_dim), dtype=self.TT, device=self.dev)
            qa.view(T, s.heads, R + s.rot_dim)[..., R:] = qd.view(T, s.heads, E)[..., s.dim:]
            m.batched_linear(qd, x.w_ukT, s.heads, a_block=E, out=qa, c_block=R + s.rot_dim)
            x.attend_latent(qa, b, out, gd, s.heads * s.vdim, s.window)
        return out.double().cpu().view(T, s.heads, s.vdim)

    def want(self, q, gate, parts):
        s = self.s
        H, D, Dv, R = s.heads, s.dim, s.vdim, s.kv_rank
        out, t = torch.zeros(q.shape[0], H, Dv, dtype=D64), 0
        for k, p0, n in parts:
            rows = self.seqs[k][0]
            ku, v = (rows[:, :R] @ self.uk.double().T).view(-1, H, D), (rows[:, :R] @ self.uv.double().T).view(-1, H, Dv)
            for i in range(p0, p0 + n):
                lo = max(0, i - s.window + 1) if s.window else 0
                for h in range(H):
                    sc = (ku[lo:i + 1, h] @ q[t, h, :D].double() + rows[lo:i + 1, R:] @ q[t, h, D:].double()) * s.scale
                    out[t, h] = O.softmax_sink(sc, self.sink[h].double()) @ v[lo:i + 1, h]
                t += 1
        return out if gate is None else out * torch.sigmoid(gate.double().view(out.shape))


def _bf(g, *shape, scale=1.0):
    return (torch.randn(*shape, generator=g) * scale).to(torch.bfloat16).float()


SIZES = [(4, 16, 8, 32, 32, 21), (3, 8, 16, 24, 48, 0), (17, 32, 16, 32, 112, 60), (2, 64, 64, 128, 256, 50), (1, 128, 64, 96, 512, 0), (5, 40, 0, 64, 64, 33), (2, 8, 8, 8, 16, 1), (33, 16, 16, 16, 80, 5),
         (2, 192, 64, 64, 64, 40), (2, 16, 8, 16, 600, 30)]


@pytest.mark.gpu
@pytest.mark.parametrize("expanded", [True, False], ids=["expanded", "cached_rows"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H,D,Dr,Dv,R,window", SIZES)
def test_latent_attention_over_portions_and_single_rows(dev, H, D, Dr, Dv, R, window, dtype, expanded):
    """portions (one ends in the middle of a page and a segment) and single rows of sequences of unequal length over shuffled pages whose unused slots hold NaN; the bf16 forms
    run on the matrix cores where their tiles cover the size"""
    rig = LatentRig(dev, dtype, H, D, Dr, Dv, R, window, seed=H + R)
    assert rig.x.mfma_prompt == (dtype == "bfloat16") and rig.x.mfma_decode == (dtype == "bfloat16" and R <= 512)
    g = rig.g
    for P in (150, 37, 5):
        rig.add(_bf(g, P, R + Dr))
    for parts in ([(0, 20, 130), (1, 36, 1), (2, 0, 5)], [(0, 149, 1), (1, 36, 1), (2, 4, 1)], [(1, 7, 2)]):
        T = sum(n for _, _, n in parts)
        if expanded and T == len(parts):
            continue
        q, gate = _bf(g, T, H, D + Dr), torch.randn(T, H * Dv, generator=g)
        got, want = rig.run(q, gate, parts, expanded), rig.want(q, gate, parts)
        assert rel(got, want) < (2e-5 if dtype == "float32" else 8e-3), parts
        got, want = rig.run(q, None, parts, expanded), rig.want(q, None, parts)
        assert rel(got, want) < (2e-5 if dtype == "float32" else 8e-3), parts


@pytest.mark.gpu
@pytest.mark.parametrize("form", ["expanded", "cached_rows", "single_rows"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("window", [7, 8, 24, 64, 0])
def test_planted_keys_at_the_window_edges(dev, window, dtype, form):
    """one key per query scores far above the rest: the oldest key of the window (must be read), the one before it (must not be), the query itself, the first slot of a page;
    the key part carries the score and the latent names the position, so that the output says which position was read"""
    H, D, Dr, Dv, R, P = 2, 8, 64, 8, 16, 96
    rig = LatentRig(dev, dtype, H, D, Dr, Dv, R, window, scale=1.0, seed=window)
    g = rig.g
    rig.uv.zero_()
    for h in range(H):
        rig.uv[h * Dv, 0], rig.uv[h * Dv + 1, 1], rig.uv[h * Dv + 2, 2] = 1.0, 1.0, 1.0     # values: position / 16, position % 16, one
    rig.x.w_uv = rig.uv.view(H, Dv, R).to(dev, rig.TT)
    rig.sink[:] = torch.tensor([-30.0, 4.0])
    rig.x.sink = rig.sink.float().to(dev)
    rows = torch.zeros(P, R + Dr)
    pos = torch.arange(P)
    rows[:, 0], rows[:, 1], rows[:, 2] = (pos // 16).float(), (pos % 16).float(), 1.0
    # key parts that are far apart: +- 1 patterns of the position's bits, repeated
    code = torch.stack([torch.randint(0, 2, (Dr,), generator=torch.Generator().manual_seed(100 + p)).float() * 2 - 1 for p in range(P)])
    rows[:, R:] = code
    rig.add(rows)
    q0 = 40
    T = P - q0
    q = torch.zeros(T, H, D + Dr)
    targets = []
    for r in range(T):
        i = q0 + r
        lo = max(0, i - window + 1) if window else 0
        tgt = [lo, lo - 1, i, (i // 8) * 8][r % 4]
        targets.append(tgt)
        q[r, :, D:] = code[max(tgt, 0)] * (1.0 if tgt >= 0 else -1.0)       # score 64 on the planted key, at most about 40 elsewhere
    gate = torch.zeros(T, H * Dv)
    if form == "single_rows":
        got = torch.cat([rig.run(q[r:r + 1], gate[r:r + 1], [(0, q0 + r, 1)], False) for r in range(T)])
    else:
        got = rig.run(q, gate, [(0, q0, T)], form == "expanded")
    want = rig.want(q, gate, [(0, q0, T)])
    assert float((got - want).abs().max()) < (1e-4 if dtype == "float32" else 0.03)
    inside = outside = 0
    for r in range(T):
        i = q0 + r
        lo = max(0, i - window + 1) if window else 0
        read = float(16 * got[r, 0, 0] / got[r, 0, 2] + got[r, 0, 1] / got[r, 0, 2])
        if targets[r] >= lo and targets[r] >= 0:
            assert abs(read - targets[r]) < 0.3, (r, targets[r], read)
            inside += targets[r] == lo
        else:
            assert read >= lo - 0.3, (r, targets[r], read)      # nothing from before the window
            outside += 1
    assert inside >= 3 and (outside >= 3 or not window)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_sink_alone_takes_the_weight_once(dev, dtype):
    """queries that match nothing next to a large, a small and no sink: n keys weigh n / (n + e^sink) together, in portions and in single rows dealt to several workgroups"""
    H, D, Dr, Dv, R, P = 3, 8, 8, 8, 16, 300
    rig = LatentRig(dev, dtype, H, D, Dr, Dv, R, 0, seed=3)
    rig.sink[:] = torch.tensor([5.5, 0.0, -40.0])
    rig.x.sink = rig.sink.float().to(dev)
    rig.add(_bf(rig.g, P, R + Dr))
    q = torch.zeros(4, H, D + Dr)
    v = (rig.seqs[0][0][:, :R] @ rig.uv.double().T).view(P, H, Dv)
    for parts, expanded in (([(0, P - 4, 4)], True), ([(0, P - 4, 4)], False), ([(0, P - 1, 1)], False), ([(0, 0, 1)], False)):
        n = parts[0][2]
        got = rig.run(q[:n], None, parts, expanded)
        for r in range(n):
            k = parts[0][1] + r + 1
            for h in range(H):
                want = v[:k, h].mean(0) * k / (k + math.exp(float(rig.sink[h])))
                assert float((got[r, h] - want).abs().max()) < (1e-5 if dtype == "float32" else 4e-3 * max(1.0, float(want.abs().max()))), (parts, r, h)   # (bf16: joined sums and result, each rounded once)


@pytest.mark.gpu
def test_matrix_core_weights_keep_their_low_bits(dev):
    """bf16 attention whose value is one large column of alternating sign with nearly equal weights: the sum cancels to what the weights' low bits say, so weights rounded to bf16 would be
    off by orders of magnitude more than the f32 arithmetic allows"""
    H, D, Dr, Dv, R, P = 1, 8, 8, 8, 16, 64
    rig = LatentRig(dev, "bfloat16", H, D, Dr, Dv, R, 0, scale=1.0, seed=9)
    rig.sink[:] = -60.0
    rig.x.sink = rig.sink.float().to(dev)
    rows = torch.zeros(P, R + Dr)
    rows[:, 0] = (torch.arange(P) % 2).float() * 2 - 1
    rows[:, R] = torch.arange(P).float() / 4096
    rig.uv.zero_()
    rig.uv[0, 0] = 1.0
    rig.x.w_uv = rig.uv.view(H, Dv, R).to(dev, rig.TT)
    rig.add(rows.to(torch.bfloat16).float())
    q = torch.zeros(2, H, D + Dr)
    q[:, 0, D] = 1.0
    want = rig.want(q, None, [(0, P - 2, 2)])
    for parts, expanded in (([(0, P - 2, 2)], True),):
        got = rig.run(q, None, parts, expanded)
        assert float((got[1, 0, 0] - want[1, 0, 0]).abs()) < 2e-6 and 1e-5 < float(want[1, 0, 0].abs()) < 1e-3
    got = rig.run(q[1:], None, [(0, P - 1, 1)], False)
    assert float((got[0, 0, 0] - want[1, 0, 0]).abs()) < 2e-6


# ---------------------------------------------------------------------------------------------------------------- mixers and feed-forwards alone (GPU)
def _one_layer(layer, dev, t_len=90, seed=1, dtype="float32", **kw):
    cfg = config([layer], **kw)
    w = weights(cfg, seed)
    t = toks(t_len, cfg["vocab"], seed + 100)
    want = logits_of(cfg, f64(w), t)
    sv = Served(cfg, w, dev, dtype)
    got = sv.step([(1, t[:t_len - 12])]) + sv.step([(1, t[t_len - 12:t_len - 9])]) + [sv.step([(1, [x])])[0] for x in t[t_len - 9:]]
    return torch.cat(got), want


@pytest.mark.gpu
@pytest.mark.parametrize("dtype,bar", [("float32", 3e-5), ("bfloat16", 4e-2)])
@pytest.mark.parametrize("kw", [dict(), dict(heads=1, dim=64, vdim=64), dict(heads=6, dim=7, vdim=5, tau=1.0), dict(heads=2, dim=128, vdim=16, tau=16.0), dict(heads=3, dim=40, vdim=130),
                                dict(heads=8, dim=32, vdim=32, mlp=None)])
def test_gla_mixer_alone(dev, kw, dtype, bar):
    got, want = _one_layer(gla(**kw), dev, t_len=150, dtype=dtype)
    assert close(got, want, bar)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype,bar", [("float32", 3e-5), ("bfloat16", 4e-2)])
@pytest.mark.parametrize("kw", [dict(), dict(heads=8, dim=32, rot_dim=32, vdim=32, kv_rank=64, q_rank=16, size=32), dict(heads=3, dim=10, rot_dim=6, vdim=7, kv_rank=11, q_rank=9, size=5), dict(size=0),
                                dict(scaling=None), dict(heads=2, dim=64, rot_dim=16, vdim=128, kv_rank=16, q_rank=40, size=64), dict(size=1), dict(size=1000, mlp=None), dict(rot_dim=2, scaling=(8.0, 4.0, 1.0, 16)),
                                dict(heads=20, dim=8, rot_dim=24, vdim=16, kv_rank=96, size=30)])
def test_latent_mixer_alone(dev, kw, dtype, bar):
    got, want = _one_layer(lat(**kw), dev, t_len=120, dtype=dtype)
    assert close(got, want, bar)


@pytest.mark.gpu
@pytest.mark.parametrize("f", [moe(6, 2, 24), moe(16, 4, 40), moe(3, 3, 7), moe(9, 1, 130), moe(1, 1, 8), dense(56), dense(7)])
def test_feed_forwards_alone_at_prompt_and_decode_sizes(dev, f):
    """70 rows (grouped products over expert-sorted rows) and 1 - 3 rows (every route streams its expert's slabs)"""
    got, want = _one_layer(gla(heads=1, dim=4, vdim=4, mlp=f), dev, t_len=82)
    assert rel(got, want) < 3e-5


@pytest.mark.gpu
@pytest.mark.parametrize("dtype,bar", [("float32", 5e-5), ("bfloat16", 6e-2)])
def test_sharp_attention_needs_the_window_the_sink_the_rotation_and_the_gate(dev, dtype, bar):
    """queries and keys scaled until most rows put their weight on few keys: a restatement with a window one off, without the sink, without the frequency ramp or its multiplier is far away;
    the served model is not"""
    layer = lat(heads=2, dim=8, rot_dim=16, vdim=8, kv_rank=16, q_rank=16, size=13, scale=0.8, scaling=(8.0, 4.0, 1.0, 32), mlp=None)
    cfg = config([layer])
    w = weights(cfg, 21)
    w["l0.mix.uq"] = (w["l0.mix.uq"].float() * 2).to(torch.bfloat16)
    w["l0.mix.sink"] = torch.tensor([6.0, 1.0], dtype=torch.bfloat16)
    t = toks(200, cfg["vocab"], 22)
    wd = f64(w)
    want = logits_of(cfg, wd, t)
    sv = Served(cfg, w, dev, dtype)
    got = sv.step([(1, t[:150])]) + [sv.step([(1, [x])])[0] for x in t[150:]]
    assert close(torch.cat(got), want, bar)

    def changed(f):
        c = json.loads(json.dumps(cfg))
        f(c["layers"][0]["mixer"])
        return rel(logits_of(c, wd, t), want)
    for size in (12, 14):
        assert changed(lambda m: m["mask"].__setitem__("size", size)) > 0.05
    assert changed(lambda m: m["rot"].pop("scaling")) > 0.05 and changed(lambda m: m["rot"]["scaling"].__setitem__("factor", 2.0)) > 0.02
    assert rel(logits_of(cfg, dict(wd, **{"l0.mix.sink": wd["l0.mix.sink"] - 60.0}), t), want) > 0.02
    assert rel(logits_of(cfg, dict(wd, **{"l0.mix.g": wd["l0.mix.g"] * 0}), t), want) > 0.05


@pytest.mark.gpu
def test_slow_decays_carry_the_first_tokens_across_a_long_prompt_and_decoding(dev):
    """decays close to one: the logits of the last rows depend on the first tokens (the restatement fed another beginning is far away), over portions and 300 single rows"""
    cfg = config([gla(mlp=None, tau=16.0), gla(heads=2, dim=8, vdim=16, tau=16.0, mlp=None)])
    w = weights(cfg, 31, slow=True)
    wd = f64(w)
    t = toks(420, cfg["vocab"], 32)
    want = logits_of(cfg, wd, t)
    other = logits_of(cfg, wd, toks(6, cfg["vocab"], 33) + t[6:])
    assert rel(other[-40:], want[-40:]) > 1e-3
    sv = Served(cfg, w, dev, max_tokens=448)
    got = sv.step([(1, t[:63])]) + sv.step([(1, t[63:65])]) + sv.step([(1, t[65:120])]) + [sv.step([(1, [x])])[0] for x in t[120:]]
    assert rel(torch.cat(got), want) < 5e-5


@pytest.mark.gpu
@pytest.mark.parametrize("dtype,bar", [("float32", 5e-5), ("bfloat16", 4e-2)])
@pytest.mark.parametrize("size", [0, 600, 300, 70])
def test_long_decoding_with_keys_dealt_to_several_workgroups(dev, size, dtype, bar):
    """single-row steps over hundreds of keys, two sequences of unequal length, windows that pass over decoded tokens"""
    cfg = config([lat(heads=4, dim=16, rot_dim=8, vdim=8, kv_rank=32, q_rank=16, size=size, scale=0.5, mlp=None)])
    w = weights(cfg, 41)
    wd = f64(w)
    ta, tb = toks(640, cfg["vocab"], 42), toks(290, cfg["vocab"], 43)
    wa, wb = logits_of(cfg, wd, ta), logits_of(cfg, wd, tb)
    sv = Served(cfg, w, dev, dtype, max_tokens=1024)
    sv.step([(1, ta[:560]), (2, tb[:210])])
    ga, gb = zip(*(sv.step([(1, [ta[560 + i]]), (2, [tb[210 + i]])]) for i in range(80)))
    assert close(torch.cat(ga), wa[560:], bar) and close(torch.cat(gb), wb[210:], bar)


@pytest.mark.gpu
def test_first_tokens_see_zeros_not_the_slots_former_owner(dev):
    """two slots, four requests one after the other: states of finished requests stay in the slots; a new request must not read them"""
    cfg = config([gla(), lat(), gla(tau=1.0)])
    w = weights(cfg, 23, slow=True)
    sv = Served(cfg, w, dev, max_tokens=128, slots=2)
    wd = f64(w)
    for r in range(1, 5):
        t = toks(40 + r, cfg["vocab"], 30 + r)
        want = logits_of(cfg, wd, t)
        got = sv.step([(r, t[:1])]) + sv.step([(r, t[1:3])]) + sv.step([(r, t[3:])])
        assert rel(torch.cat(got), want) < 5e-5, r
        sv.end(r)


# ---------------------------------------------------------------------------------------------------------------- whole models (GPU)
@pytest.mark.gpu
@pytest.mark.parametrize("dtype,bar", [("float32", 5e-5), ("bfloat16", 4e-2)])
def test_whole_prompt_every_layer(dev, dtype, bar):
    cfg = config(STACK)
    w = weights(cfg, 5)
    sv = Served(cfg, w, dev, dtype)
    t = toks(150, cfg["vocab"], 14)
    want, after, _ = O.forward(cfg, f64(w), t)
    sv.m.trace_layers = []
    got = sv.step([(1, t)])[0]
    assert len(sv.m.trace_layers) == len(STACK) and sv.m.has_recurrent_state and sv.m.has_paged_kv
    for i, (a, b) in enumerate(zip(sv.m.trace_layers, after)):
        assert close(a.double().cpu(), b, bar), f"residual stream after layer {i}"
    assert close(got, want, bar)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype,bar", [("float32", 5e-5), ("bfloat16", 4e-2)])
def test_portions_and_decoding_equal_the_whole_prompt(dev, dtype, bar):
    """the same 200 tokens: whole; in portions of changing sizes down to two tokens and single tokens; token by token from the start"""
    cfg = config(STACK)
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
    got = [sv.step([(3, [x])])[0] for x in t[:100]]
    assert close(torch.cat(got), want[:100], bar)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype,bar", [("float32", 5e-5), ("bfloat16", 4e-2)])
def test_mixed_batches_with_reused_pages_and_slots(dev, dtype, bar):
    """five requests of unequal length through a pool of 192 tokens and three slots: portions beside single tokens, a request left out of a step, pages and slots of finished
    requests taken by later ones -- every row against the request alone in the restatement"""
    cfg = config(STACK)
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
    """one head, one expert, windows of one position, sizes equal to the width, tau 1, one-token prompts, an embedding scale of one"""
    for layers, kw in (([gla(heads=1, dim=24, vdim=24, tau=1.0, mlp=moe(1, 1, 24)), lat(heads=1, dim=24, rot_dim=24, vdim=24, kv_rank=24, q_rank=24, size=24, mlp=dense(24))],
                        dict(width=24, vocab=24, scale=1.0)),
                       ([gla(heads=2, dim=1, vdim=1, mlp=moe(2, 1, 1)), lat(heads=2, dim=1, rot_dim=2, vdim=1, kv_rank=1, q_rank=1, size=1, mlp=dense(1)),
                         lat(heads=1, dim=2, rot_dim=2, vdim=1, kv_rank=2, q_rank=1, size=2, mlp=None)], dict(width=8, vocab=5))):
        cfg = config(layers, **kw)
        w = weights(cfg, 9, rank=1)
        t = toks(40, cfg["vocab"], 17)
        want = logits_of(cfg, f64(w), t)
        sv = Served(cfg, w, dev)
        assert rel(sv.step([(1, t[:1])])[0], want[:1]) < 5e-5
        got = sv.step([(2, t[:1])]) + sv.step([(2, t[1:3])]) + sv.step([(2, t[3:])])
        assert rel(torch.cat(got), want) < 5e-5


@pytest.mark.gpu
@pytest.mark.parametrize("dtype,bar", [("float32", 5e-5), ("bfloat16", 5e-2)])
def test_sizes_off_every_vector_width(dev, dtype, bar):
    """width, vocabulary, head sizes, ranks and feed-forward sizes that no 16-byte load divides: the element-wise paths of every kernel, prompt and decode"""
    cfg = config([gla(heads=3, dim=11, vdim=13, mlp=moe(5, 2, 27)), lat(heads=3, dim=7, rot_dim=6, vdim=5, kv_rank=21, q_rank=15, size=11, mlp=dense(15)),
                  gla(heads=1, dim=33, vdim=70, tau=2.5, mlp=moe(3, 2, 9))], vocab=77, width=50)
    w = weights(cfg, 13, rank=3)
    t = toks(100, cfg["vocab"], 18)
    want = logits_of(cfg, f64(w), t)
    sv = Served(cfg, w, dev, dtype)
    got = sv.step([(1, t[:67])]) + sv.step([(1, t[67:90])]) + [sv.step([(1, [x])])[0] for x in t[90:]]
    assert close(torch.cat(got), want, bar)


@pytest.mark.gpu
@pytest.mark.parametrize("block_size", [8, 16, 12])
def test_other_page_sizes(dev, block_size):
    """pages that the matrix-core tiles cross in other places, and one they do not take (12 tokens: the general kernels)"""
    cfg = config(STACK)
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
    from mistralrs_amd.hybrid import HybridDecoder, kebisun_spec
    from mistralrs_amd.sampler import SequenceSampler
    from mistralrs_amd.scheduler import Sequence
    cfg = config([lat(), gla(), lat(size=9, mlp="moe")])
    w = weights(cfg, 10)
    m = HybridDecoder(kebisun_spec(cfg), dev, "float32", num_blocks=12, block_size=32, state_slots=3)
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
    cfg = config(STACK)
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
    cfg = config([lat(), gla(mlp=None), lat(size=9, mlp="moe"), gla()])
    w = weights(cfg, 12)
    folder = tmp_path / "model"
    folder.mkdir()
    (folder / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in w.items()}, str(folder / "model.safetensors"))
    assert registry.architecture_of(str(folder)) == "Kebisun"
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
