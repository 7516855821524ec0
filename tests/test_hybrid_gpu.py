"""The hybrid decoder (softmax attention, decayed linear attention, mixtures of experts) on the GPU against oracle/hybrid.py:
every mechanism alone, then whole models in every way of cutting and batching the tokens."""
import numpy as np
import pytest
import torch

from omniserve_amd.models.base import EngineModel
from oracle import hybrid
from tests.hybrid_util import (attention, config, cuts, errors, lightning, moe, random_state, random_tokens, run_alone, to_numpy)

pytestmark = pytest.mark.gpu
F32, BF16 = torch.float32, torch.bfloat16
TOL = {F32: 3e-5, BF16: 2.5e-2}
DTYPES = [F32, BF16]
DEV = torch.device("cuda:0")


# ---------------------------------------------------------------------------------------------------------------
# one mixer alone: h in, output out, through the cache
# ---------------------------------------------------------------------------------------------------------------
class OneMixer(EngineModel):
    """A mixer with what the cache and the batch builder ask a model for."""
    vocab = 1

    def __init__(self, layer, width, dtype, seed, weights=None, mixes=False):
        from omniserve_amd.backend.lm import lm_ops
        from omniserve_amd.models import layers as L
        from omniserve_amd.models.bobavik import _mixer
        self.dtype, self.device, self.width, self.layer = dtype, DEV, width, layer
        self.state = {k: v for k, v in random_state(config([layer], width=width), seed).items()}
        self.state.update({"l0.mix." + k: v for k, v in (weights or {}).items()})
        w = L.Weights(self.state, DEV, dtype).under("l0.mix.")
        spec = _mixer(layer["type"], layer["mixer"])
        self.soft = layer["type"] == "attention"
        self.mixer = L.Attention(spec, w, lm_ops(dtype), width, mixes) if self.soft else L.LinearAttention(spec, w, lm_ops(dtype), width, 1e-5)
        self.W = L.pad64(width)

    def kv_shapes(self):
        return [self.mixer.cache_shape()] if self.soft else []

    def state_shapes(self):
        return [] if self.soft else self.mixer.state_shapes()

    def window(self):
        return self.layer["mixer"]["mask"]["size"] if self.soft else 1

    def linear_workgroups(self):
        return 0 if self.soft else self.mixer.s.heads * self.mixer.dv // 64

    def new_cache(self, tokens=4096, slots=3):
        from omniserve_amd.engine.cache import Cache
        return Cache(self, tokens // 64, slots, DEV)

    def run(self, h, sizes, cache=None, v_first=None, seg_len=None):
        """h [T, width] (numpy) -> the mixer's output, the sequence cut into portions of `sizes`"""
        from omniserve_amd.engine.batch import BatchBuilder, Entry
        cache, builder = cache or self.new_cache(), BatchBuilder(self, DEV)
        if seg_len:
            builder._segment_len = lambda portions: seg_len
        seq, at, out = cache.open(), 0, []
        for n in cuts(len(h), sizes):
            cache.reserve(seq, n)
            b, _ = builder.build([Entry(seq, [0] * n, [])])
            x = torch.zeros((n, self.W), dtype=self.dtype, device=DEV)
            x[:, :self.width] = torch.from_numpy(h[at:at + n]).to(DEV, self.dtype)
            if self.soft:
                vf = None
                if v_first is not None:
                    m = self.layer["mixer"]
                    vf = torch.zeros((n, m["kv_heads"], self.mixer.dv), dtype=self.dtype, device=DEV)
                    vf[..., :m["vdim"]] = torch.from_numpy(v_first[at:at + n]).to(DEV, self.dtype)
                    vf = vf.view(n, -1)
                y, _ = self.mixer(x, b, cache.kv[0], vf)
            else:
                y = self.mixer(x, b, cache.state[0])
            cache.advance(seq, n)
            out.append(y[:, :self.width].float().cpu())
            at += n
        cache.close(seq)
        return torch.cat(out).numpy()

    def oracle(self, h, v_first=None, **changed):
        w = hybrid.under(to_numpy(self.state), "l0.mix.")
        m = dict(self.layer["mixer"], **changed)
        if self.soft:
            return hybrid.attention_mixer(h, w, m, v_first)[0]
        return hybrid.lightning_mixer(h, w, m, 1e-5)


def inputs(T, width, seed):
    x = np.random.default_rng(seed).standard_normal((T, width))
    return torch.from_numpy(x).bfloat16().double().numpy()      # the same values in both formats


ATTENTION = {
    "grouped": attention(heads=6, kv_heads=2, dim=48, vdim=40, window=37, rot=32),
    "one kv head, 20 query heads": attention(heads=20, kv_heads=1, dim=32, vdim=64, window=100, rot=32, scaling=False),
    "window 1": attention(heads=2, kv_heads=2, dim=24, vdim=24, window=1, rot=8),
    "window = page, no rotation": attention(heads=3, kv_heads=3, dim=64, vdim=96, window=64, rot=0),
    "128 / 128": attention(heads=4, kv_heads=2, dim=128, vdim=128, window=130, rot=128),
    "256 / 64, wide window": attention(heads=2, kv_heads=1, dim=200, vdim=16, window=1000, rot=64),
    "64 / 256": attention(heads=2, kv_heads=2, dim=16, vdim=256, window=65, rot=16),
    "256 / 256": attention(heads=2, kv_heads=1, dim=256, vdim=256, window=90, rot=128),
}
LINEAR = {
    "unequal sizes": lightning(heads=3, dim=40, vdim=72),
    "one head": lightning(heads=1, dim=64, vdim=16, decay=[0.9]),
    "decays 0 and 1": lightning(heads=2, dim=32, vdim=64, decay=[0.0, 1.0]),
    "128 / 128": lightning(heads=2, dim=128, vdim=128, decay=[0.999, 0.6]),
    "256 / 200": lightning(heads=2, dim=256, vdim=200, decay=[1.0, 0.97]),
}


@pytest.mark.parametrize("dtype", DTYPES, ids=str)
@pytest.mark.parametrize("name", list(ATTENTION))
def test_attention_mixer(name, dtype):
    m = OneMixer(ATTENTION[name], 96, dtype, seed=1)
    h = inputs(333, 96, 2)
    want = m.oracle(h)
    for sizes in ([333], [200, 2, 64, 3, 1, 1, 63], [1]):
        e = errors(m.run(h, sizes), want)
        assert e.max() < TOL[dtype], (sizes, e.argmax(), e.max())


@pytest.mark.parametrize("dtype", DTYPES, ids=str)
@pytest.mark.parametrize("name", list(LINEAR))
def test_linear_attention_mixer(name, dtype):
    m = OneMixer(LINEAR[name], 96, dtype, seed=3)
    h = inputs(450, 96, 4)
    want = m.oracle(h)
    for sizes, seg in (([450], None), ([450], 64), ([450], 128), ([31, 2, 64, 1, 1, 130], 64), ([2], None), ([1], None)):
        e = errors(m.run(h, sizes, seg_len=seg), want)
        assert e.max() < TOL[dtype], (sizes, seg, e.argmax(), e.max())


@pytest.mark.parametrize("dtype", DTYPES, ids=str)
def test_value_mixing(dtype):
    layer = attention(heads=4, kv_heads=2, dim=32, vdim=40, window=50, rot=32)
    m = OneMixer(layer, 96, dtype, seed=5, mixes=True)
    h, vf = inputs(150, 96, 6), inputs(150, 80, 7).reshape(150, 2, 40)
    want = m.oracle(h, v_first=vf)
    assert errors(m.oracle(h), want).min() > 4 * TOL[dtype]            # it matters at every position
    for sizes in ([150], [70, 2, 1, 1], [1]):
        assert errors(m.run(h, sizes, v_first=vf), want).max() < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES, ids=str)
@pytest.mark.parametrize("window", [63, 64, 65, 128, 200])
def test_one_key_stands_out_at_the_edge_of_the_window(window, dtype):
    """q and k are the same projection of the first half of h, values come from the second half: a key whose first half equals
    the query's scores as high as the query's own, everything else is negligible.  It sits just inside, just outside or at a page
    border of the window."""
    W, H, D = 96, 2, 32
    layer = attention(heads=H, kv_heads=H, dim=D, vdim=32, window=window, rot=0, scale=0.5, v_mix=False)
    g = torch.Generator().manual_seed(8)
    wq = torch.zeros((H * D, W))
    wq[:, :48] = torch.randn((H * D, 48), generator=g) / 48 ** 0.5
    wv = torch.zeros((H * 32, W))
    wv[:, 48:] = torch.randn((H * 32, 48), generator=g) / 48 ** 0.5
    m = OneMixer(layer, W, dtype, seed=9, weights={"q": (1.6 * wq).bfloat16(), "k": (1.6 * wq).bfloat16(), "v": wv.bfloat16()})
    T = 520
    h = inputs(T, W, 10)
    shows = []
    for i in (window - 1, window, 255, 256, 257, 319, 400, 511, 519):
        for j in (i - window + 1, i - window):
            if j < 0 or j == i:
                continue
            x = h.copy()
            x[j, :48] = x[i, :48]
            want = m.oracle(x)[i:i + 1]
            off = m.oracle(x, mask={"size": window + (1 if j == i - window else -1)})[i:i + 1]
            shows.append(errors(off, want)[0])
            for sizes in ([T], [i] + [1] * (T - i)):
                e = errors(m.run(x[:i + 1], sizes)[i:i + 1], want)[0]
                assert e < 2 * TOL[dtype], (i, j, sizes[0], e)
    assert min(shows) > 8 * TOL[dtype], shows


@pytest.mark.parametrize("dtype", DTYPES, ids=str)
def test_far_key_of_the_recurrent_state(dtype):
    """one key of large weight far back; q of the asking token points at it"""
    W = 96
    layer = lightning(heads=2, dim=32, vdim=32, decay=[0.9995, 0.999])
    state = random_state(config([layer], width=W), 11)
    m = OneMixer(layer, W, dtype, seed=11, weights={"k": state["l0.mix.q"]})
    h = inputs(1500, W, 12)
    h[1400] = h[3]
    h[3] *= 24.0
    want = m.oracle(h)[1400:1401]
    cut = hybrid.lightning_mixer(h[4:], hybrid.under(to_numpy(m.state), "l0.mix."), layer["mixer"], 1e-5)[1396:1397]
    assert errors(cut, want)[0] > 8 * TOL[dtype]
    for sizes in ([1401], [1400, 1], [64, 2, 300], [700, 699] + [1] * 8):
        assert errors(m.run(h[:1401], sizes)[1400:1401], want)[0] < 2 * TOL[dtype], sizes


# ---------------------------------------------------------------------------------------------------------------
# feed-forward, norms, products, routing
# ---------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES, ids=str)
@pytest.mark.parametrize("tokens", [1, 7, 16, 33, 64, 65, 300, 1200])
@pytest.mark.parametrize("kind", [dict(), dict(top=1, shared=None), dict(experts=1, top=1, ff=64, shared=64), dict(experts=5, top=5, ff=130, shared=16), dict(experts=70, top=8)], ids=str)
def test_mixture(kind, tokens, dtype):
    from omniserve_amd.backend.lm import lm_ops
    from omniserve_amd.models import layers as L
    from omniserve_amd.models.bobavik import _moe
    width, spec = 96, moe(**kind)
    state = random_state(config([dict(attention(), mlp=spec)], width=width), 13)
    ops, W = lm_ops(dtype), L.pad64(width)
    mix = L.MixtureOfExperts(_moe(spec), L.Weights(state, DEV, dtype).under("l0.mlp."), ops, width)
    h = inputs(tokens, width, 14)
    w = hybrid.under(to_numpy(state), "l0.mlp.")
    want, (ids, wt) = hybrid.mixture(h, w, spec), hybrid.route(h, w["router"], w["router.b"], spec["router"]["top"])
    x = torch.zeros((tokens, W), dtype=dtype, device=DEV)
    x[:, :width] = torch.from_numpy(h).to(DEV, dtype)
    y, experts = mix(x)
    assert np.abs(experts["experts"][0].cpu().numpy() - wt).max() < 1e-4
    r = torch.zeros((tokens, W), dtype=F32, device=DEV)
    ops.residual_norm(r, width, "layer", 1e-5, y=y, **experts)                # the weighted sum alone
    e = errors(r[:, :width].cpu().numpy(), want)
    assert e.max() < TOL[dtype], e.max()


@pytest.mark.parametrize("dtype", DTYPES, ids=str)
@pytest.mark.parametrize("width", [64, 100, 1024, 1500, 5000])
@pytest.mark.parametrize("kind", ["layer", "rms"])
def test_residual_norm(kind, width, dtype):
    from omniserve_amd.backend.lm import lm_ops
    from omniserve_amd.models.layers import pad64, padded
    ops, W, T, eps = lm_ops(dtype), pad64(width), 5, 1e-3
    g = np.random.default_rng(15)
    x, y = 30 + g.standard_normal((T, width)), torch.from_numpy(0.03 * g.standard_normal((T, width))).to(dtype).double().numpy()
    w = [1 + 0.3 * g.standard_normal(width) for _ in range(2)]
    b = [g.standard_normal(width) if kind == "layer" else None for _ in range(2)]
    f = (lambda z, i: hybrid.layer_norm(z, w[i], b[i], eps)) if kind == "layer" else (lambda z, i: hybrid.rms_norm(z, w[i], eps))
    new = x + f(y, 0)
    dev = lambda a, t=F32: None if a is None else torch.from_numpy(a).to(DEV, t)      # noqa: E731
    pv = lambda a: None if a is None else padded(dev(a), W)                           # noqa: E731
    xs, ys = padded(dev(x), T, W), padded(dev(y, dtype), T, W)
    h = torch.full((T, W), 7.0, dtype=dtype, device=DEV)
    ops.residual_norm(xs, width, kind, eps, y=ys, post=(pv(w[0]), pv(b[0])), next=(pv(w[1]), pv(b[1])), h=h)
    assert errors(xs[:, :width].cpu().numpy(), new).max() < 1e-6
    assert errors(h[:, :width].float().cpu().numpy(), f(new, 1)).max() < (2e-5 if dtype == F32 else 5e-3)
    assert not h[:, width:].any()


@pytest.mark.parametrize("dtype", DTYPES, ids=str)
@pytest.mark.parametrize("H,G,dk,dv,dims", [(4, 2, 64, 128, 64), (3, 3, 128, 64, 6), (2, 1, 256, 64, 256), (2, 2, 64, 64, 0)])
def test_rotation_and_append(H, G, dk, dv, dims, dtype):
    """q turned in place, k turned and v mixed into their page places; slot -1 stores nothing; far positions"""
    from omniserve_amd.backend.lm import lm_ops
    ops, T, g = lm_ops(dtype), 9, np.random.default_rng(23)
    pos, slot = np.array([0, 1, 2, 63, 64, 65, 500, 4095, 100]), np.array([0, 1, 2, 63, 64 * 3, 64 * 3 + 1, 130, 64 * 2 - 1, -1])
    x = torch.from_numpy(g.standard_normal((T, (H + G) * dk + G * dv))).to(DEV, dtype)
    vf = torch.from_numpy(g.standard_normal((T, G * dv))).to(DEV, dtype)
    q, k, v = (t.double().cpu().numpy() for t in x.split([H * dk, G * dk, G * dv], dim=1))
    fr = hybrid.rope_frequencies(dims, 20000.0, dict(factor=4.0, low=1.0, high=4.0, original=300))
    kc, vc = (torch.full((4, G, 64, d), 9.0, dtype=dtype, device=DEV) for d in (dk, dv))
    i32 = lambda a: torch.from_numpy(a.astype(np.int32)).to(DEV)      # noqa: E731
    ops.rope_append(x, vf, 0.3, torch.tensor(fr, dtype=F32, device=DEV), i32(pos), i32(slot), kc, vc, H, G, dk, dv)
    tol = 3e-4 if dtype == F32 else 5e-3                                 # (angles are f32: 4095 * 2^-24)
    turn = lambda a, n: hybrid.rotate_pairs(a.reshape(T, n, dk), pos, fr)                              # noqa: E731
    assert errors(x[:, :H * dk].double().cpu().numpy(), turn(q, H).reshape(T, -1)).max() < tol
    wk, wv = turn(k, G), hybrid.mix_values(v, vf.double().cpu().numpy(), 0.3).reshape(T, G, dv)
    kn, vn = (c.double().cpu().numpy() for c in (kc, vc))
    for t in range(T - 1):
        p, o = divmod(slot[t], 64)
        assert errors(kn[p, :, o], wk[t]).max() < tol and errors(vn[p, :, o], wv[t]).max() < tol
    assert (kn == 9.0).sum() == kn.size - (T - 1) * G * dk and (vn == 9.0).sum() == vn.size - (T - 1) * G * dv


@pytest.mark.parametrize("dtype", DTYPES, ids=str)
@pytest.mark.parametrize("n", [40, 64, 900, 4096])
def test_gated_rms(n, dtype):
    from omniserve_amd.backend.lm import lm_ops
    from omniserve_amd.models.layers import pad64, padded
    ops, T, C, g = lm_ops(dtype), 6, pad64(n), np.random.default_rng(24)
    o, z = (torch.from_numpy(g.standard_normal((T, n)) * s).to(dtype) for s in (1e-3, 2.0))
    w = torch.from_numpy(1 + 0.3 * g.standard_normal(n)).float()
    want = hybrid.rms_norm(o.double().numpy(), w.double().numpy(), 1e-6) * hybrid.sigmoid(z.double().numpy())
    out = padded(o, T, C).to(DEV)
    ops.gated_rms(out, out, padded(z, T, C).to(DEV), padded(w, C).to(DEV), n, 1e-6)
    assert errors(out[:, :n].float().cpu().numpy(), want).max() < (2e-6 if dtype == F32 else 4e-3) and not out[:, n:].any()


def test_argmax_takes_the_first_of_equals():
    from omniserve_amd.backend.lm import lm_ops
    z = torch.zeros((4, 5000), device=DEV)
    z[0, 4999] = z[0, 3000] = 2.0
    z[1] = -1.0
    z[2, 1023] = z[2, 1024] = 1.0
    z[3, 4200] = 9.0
    assert lm_ops(F32).argmax(z, 4200).tolist() == [3000, 0, 1023, 0]


@pytest.mark.parametrize("dtype", DTYPES, ids=str)
@pytest.mark.parametrize("m,n,k", [(1, 304, 64), (16, 1024, 192), (17, 48, 1024), (50, 25600, 128), (64, 80, 4096), (130, 144, 192),
                                   (700, 528, 320), (257, 16, 64), (1000, 32, 1024)])
def test_products(m, n, k, dtype):
    from omniserve_amd.backend.lm import lm_ops
    ops = lm_ops(dtype)
    g = torch.Generator(device="cuda").manual_seed(16)
    x, w = (torch.randn(s, generator=g, device=DEV).to(dtype) for s in ((m, k), (n, k)))
    want = (x.double() @ w.double().t()).cpu().numpy()
    assert errors(ops.matmul(x, w, out_f32=True, scale=0.5).cpu().numpy(), 0.5 * want).max() < 2e-6
    assert errors(ops.matmul(x, w).float().cpu().numpy(), want).max() < (2e-6 if dtype == F32 else 4e-3)


def test_routing_ties_and_order():
    from omniserve_amd.backend.lm import lm_ops
    ops = lm_ops(F32)
    for T in (3, 64, 65, 1000, 5000):
        g = np.random.default_rng(17)
        z = g.integers(0, 4, (T, 40)).astype(np.float32)           # many ties
        bias = g.integers(0, 2, 40).astype(np.float32)
        zt = torch.zeros((T, 48), device=DEV)
        zt[:, :40] = torch.from_numpy(z)
        wts, (off, perm, tiles, _, top) = ops.route(zt, torch.from_numpy(bias).to(DEV), 40, 3)
        ids, wt = hybrid.route(np.eye(40)[np.zeros(T, int)] * 0 + z, np.eye(40), bias, 3)
        off, perm = off.cpu().numpy(), perm.cpu().numpy()
        assert np.abs(wts.cpu().numpy() - wt).max() < 1e-6
        flat = ids.reshape(-1)
        assert sorted(perm.tolist()) == list(range(3 * T))
        for e in range(40):
            assert sorted(perm[off[e]:off[e + 1]]) == np.nonzero(flat == e)[0].tolist()
        if tiles is not None:
            t = [r for r in tiles.cpu().numpy().tolist() if r[2]]
            assert t == [[e, p, min(256, off[e + 1] - p), 0] for e in range(40) for p in range(off[e], off[e + 1], 256)]


# ---------------------------------------------------------------------------------------------------------------
# whole models
# ---------------------------------------------------------------------------------------------------------------
MODELS = {
    "mixed": config([lightning(), attention(window=37), attention(window=90, heads=6, kv_heads=2, top=1, shared=None),
                     lightning(heads=2, mlp=None), attention(window=37, v_mix=False, kv_heads=4, vdim=24)]),
    "attention last of two": config([lightning(heads=1, decay=[0.97], shared=None), attention(heads=2, kv_heads=1, window=129, rot=48)],
                                    width=200, vocab=77, logit_scale=1.0, eps=1e-3),
    "recurrent only": config([lightning(), lightning(heads=2, dim=128, vdim=64, mlp=None)], width=64, vocab=130),
    "attention only": config([attention(window=70, mlp=None), attention(window=64, scaling=False, mlp=None)], width=96),
}
_cache = {}


def model_and_oracle(name, dtype, T=400):
    from omniserve_amd.models.bobavik import Bobavik
    cfg = MODELS[name]
    if name not in _cache:
        state, tokens = random_state(cfg, 18), random_tokens(cfg, T, 19)
        _cache[name] = (state, tokens, hybrid.decoder(cfg, to_numpy(state), tokens))
    state, tokens, want = _cache[name]
    if (name, dtype) not in _cache:
        _cache[name, dtype] = Bobavik.from_state(cfg, state, dtype)
    return cfg, _cache[name, dtype], tokens, want


def check(got, want, dtype, what=""):
    """f32: every position; bf16: a rounded router input may change a choice now and then, so all but a few."""
    e = errors(got, want)
    if dtype == F32:
        assert e.max() < 1e-4, (what, int(e.argmax()), e.max())
    else:
        assert np.median(e) < 0.03 and (e > 0.1).sum() <= max(2, 0.05 * e.size), (what, np.median(e), (e > 0.1).mean())


@pytest.mark.parametrize("dtype", DTYPES, ids=str)
@pytest.mark.parametrize("name", list(MODELS))
def test_model_in_portions(name, dtype):
    from omniserve_amd.engine import Engine
    cfg, model, tokens, (want, _) = model_and_oracle(name, dtype)
    engine = Engine(model, max_tokens=1024, max_seqs=2)
    for sizes in ([400], [2], [1], [63, 2, 64, 65, 3], [1, 128, 1, 1, 127], [300] + [1] * 400):
        check(run_alone(engine, tokens, sizes), want, dtype, sizes[:4])
    assert engine.cache.free_pages() == engine.cache.num_pages * bool(engine.cache.paged)


def test_residual_after_every_layer():
    from omniserve_amd.engine import Engine
    cfg, model, tokens, (_, after) = model_and_oracle("mixed", F32)
    got = {}
    model.tap = lambda i, x: got.__setitem__(i, x.cpu().numpy().copy())
    try:
        run_alone(Engine(model, max_tokens=512, max_seqs=1, use_graphs=False), tokens, [400])
    finally:
        model.tap = None
    for i in range(len(cfg["layers"])):
        assert errors(got[i], after[i]).max() < 1e-4, i


@pytest.mark.parametrize("dtype", DTYPES, ids=str)
@pytest.mark.parametrize("graphs", [True, False])
def test_unequal_requests_in_one_batch(graphs, dtype):
    """Requests of unequal length advance by portions and single tokens in the same steps, with few pages and slots, so that both
    are taken again; every one has the logits it has alone."""
    from omniserve_amd.engine import Engine, SequenceInput
    cfg, model, tokens, (want, _) = model_and_oracle("mixed", dtype)
    w = to_numpy(_cache["mixed"][0])
    lengths = [400, 5, 130, 1, 64, 260, 65, 2, 33]
    reqs = [(tokens, want)] + [(t, hybrid.decoder(cfg, w, t)[0]) for t in (random_tokens(cfg, n, 20 + n) for n in lengths[1:])]
    engine = Engine(model, max_tokens=64 * 12, max_seqs=4, use_graphs=graphs)
    rng = np.random.default_rng(21)
    todo, live, got = list(range(len(reqs))), {}, {i: [] for i in range(len(reqs))}
    while todo or live:
        while todo and len(live) < 4:
            i = todo.pop(0)
            live[i] = [engine.open(), 0]
        entries, picked = [], []
        for i, (seq, at) in live.items():
            if rng.random() < 0.15 and len(live) > 1:
                continue                                  # left out of this step
            n = min(int(rng.choice([1, 1, 1, 2, 3, 17, 64, 70])), len(reqs[i][0]) - at)
            entries.append(SequenceInput(seq, reqs[i][0][at:at + n], list(range(n))))
            picked.append((i, n))
        if not entries:
            continue
        z = engine.run(entries).cpu().numpy()
        for i, n in picked:
            got[i].append(z[:n])
            z = z[n:]
            live[i][1] += n
            if live[i][1] == len(reqs[i][0]):
                engine.close(live.pop(i)[0])
    for i, (t, ref) in enumerate(reqs):
        check(np.concatenate(got[i]), ref, dtype, "request %d" % i)


@pytest.mark.parametrize("first", [1, 2, 70])
def test_a_used_slot_starts_from_zero(first):
    """whatever a slot's state holds, a new sequence's first step does not see it -- a single token, a short or a long portion"""
    from omniserve_amd.engine import Engine
    cfg, model, tokens, (want, _) = model_and_oracle("recurrent only", F32)
    engine = Engine(model, max_tokens=1024, max_seqs=1)
    for s in engine.cache.state:
        s.fill_(float("nan"))
    check(run_alone(engine, tokens[:140], [first, 1, 64]), want[:140], F32)


def test_wanted_rows_come_in_the_order_asked_for():
    from omniserve_amd.engine import Engine, SequenceInput
    cfg, model, tokens, (want, _) = model_and_oracle("attention only", F32)
    engine = Engine(model, max_tokens=1024, max_seqs=4)
    a, b, c = engine.open(), engine.open(), engine.open()
    z = engine.run([SequenceInput(a, tokens[:1], [0]), SequenceInput(b, tokens[:9], [8, 2]), SequenceInput(c, tokens[:5], [])])
    check(z.cpu().numpy(), want[[0, 8, 2]], F32)
    assert engine.run([SequenceInput(c, tokens[5:7], [])]) is None
    z = engine.run([SequenceInput(c, tokens[7:8], []), SequenceInput(b, tokens[9:10], [0]), SequenceInput(a, tokens[1:2], [0])])
    check(z.cpu().numpy(), want[[9, 1]], F32)


@pytest.mark.parametrize("name", ["mixed", "recurrent only"])
def test_greedy_generation_through_the_scheduler(name):
    """Few pages and a small token budget: prompts run in portions beside decoding requests, some are put back and recomputed.
    Every generated token is the oracle's choice after the same tokens (or within rounding of it)."""
    from omniserve_amd.engine import Engine, SamplingParams
    cfg, model, tokens, _ = model_and_oracle(name, F32)
    prompts = [tokens[:n] for n in (150, 3, 1, 64, 90)]
    engine = Engine(model, max_tokens=64 * 6, max_seqs=3, max_batch_tokens=48)
    outs = engine.generate(prompts, [SamplingParams(max_tokens=n) for n in (40, 150, 70, 5, 1)])
    w = to_numpy(_cache[name][0])
    for p, o, n in zip(prompts, outs, (40, 150, 70, 5, 1)):
        assert o.prompt == p and len(o.tokens) == n and o.finish_reason == "length"
        z = hybrid.decoder(cfg, w, p + o.tokens)[0][len(p) - 1:-1]
        best = z.max(axis=1)
        assert (best - z[np.arange(n), o.tokens] <= 1e-3 * np.abs(z).max()).all()
    assert engine.cache.free_slots() == 3


def test_long_decoding_gives_pages_back_and_stays_exact():
    """900 tokens decoded one by one in a pool that holds fewer: pages behind every window are used again."""
    from omniserve_amd.engine import Engine, SequenceInput
    cfg, model, _, _ = model_and_oracle("mixed", F32)
    tokens = random_tokens(cfg, 900, 22)
    want = hybrid.decoder(cfg, to_numpy(_cache["mixed"][0]), tokens)[0]
    engine = Engine(model, max_tokens=256, max_seqs=1)
    seq, out = engine.open(), []
    for t in tokens:
        out.append(engine.run([SequenceInput(seq, [t], [0])]).cpu().numpy())
    check(np.concatenate(out), want, F32)
    assert seq.pages == 15 and seq.released >= 12


def test_captured_steps_replay_like_eager_ones():
    from omniserve_amd.engine import Engine, SequenceInput
    cfg, model, tokens, _ = model_and_oracle("mixed", BF16)
    out = []
    for graphs in (True, False):
        engine = Engine(model, max_tokens=2048, max_seqs=8, use_graphs=graphs)
        seqs = [engine.open() for _ in range(5)]
        z = [engine.run([SequenceInput(s, tokens[i:i + 40 + i], [39 + i]) for i, s in enumerate(seqs)]).clone()]
        for k in range(12):
            live = seqs[: 5 if k % 3 else 3]
            z.append(engine.run([SequenceInput(s, [tokens[k + 7 * i]], [0]) for i, s in enumerate(live)]).clone())
            torch.zeros((1 << 20,), device=DEV).sum().item()          # the caller's own work between replays
        out.append(torch.cat(z).cpu().numpy())
    assert np.array_equal(out[0], out[1])


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_replay(tmp_path, dtype):
    import json
    import os
    import subprocess
    import sys
    from omniserve_amd import ckpt
    cfg, _, tokens, (want, _) = model_and_oracle("mixed", F32)
    ckpt.save_checkpoint(_cache["mixed"][0], str(tmp_path / "m"), cfg)
    (tmp_path / "o").mkdir()
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": tokens[:70], "want": [69, 3]}, {"id": "b", "tokens": tokens[:1], "want": [0]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": tokens[70:71], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": tokens[1:3], "want": [1]}, {"id": "a", "tokens": tokens[71:72], "want": [0]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "c", "tokens": tokens[:2], "want": [1]}], "end": ["b", "c"]}]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", str(tmp_path / "m"), "--dtype", dtype, "--out",
                        str(tmp_path / "o"), "--max-tokens", "256"], input="".join(json.dumps(s) + "\n" for s in steps), text=True,
                       capture_output=True, timeout=110)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done %d" % i for i in range(4)]
    for i, rows in ((0, [69, 3, 0]), (2, [2, 71]), (3, [1])):
        got = np.fromfile(str(tmp_path / "o" / ("%d.f32" % i)), "<f4").reshape(len(rows), -1)
        assert errors(got, want[rows]).max() < (1e-4 if dtype == "float32" else 0.15)
    assert not (tmp_path / "o" / "1.f32").exists()
