"""GPU: every kernel of the mixers library against the plain fp64 functions of oracle/vozalorn_ref.py, in both storage types, at sizes
around the tiles' edges."""
import math

import numpy as np
import pytest
import torch

from oracle import vozalorn_ref as V
from vozalorn_util import rel_err

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
BF, F32 = torch.bfloat16, torch.float32
TYPES = pytest.mark.parametrize("dt", [BF, F32], ids=["bf16", "f32"])


@pytest.fixture(scope="module")
def ops():
    from evo_amd.ops import default_ops
    return default_ops()


@pytest.fixture(params=[True, False], ids=["mfma", "any"])
def mfma(request, ops):
    ops.mixer_mfma = request.param
    yield request.param
    ops.mixer_mfma = True


def rnd(*shape, seed=0, dt=F32, scale=1.0):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(*shape, generator=g) * scale).to(dt)


def tol(dt, bf=6e-3, f=5e-6):
    return bf if dt == BF else f


# ------------------------------------------------------------------------------------------------ stream kernels
@TYPES
@pytest.mark.parametrize("M,D", [(1, 8), (3, 100), (5, 192), (70, 4096), (2, 4104), (2, 5001), (33, 1032)])
def test_stream_kernels(ops, dt, M, D):
    x, y, w = rnd(M, D, seed=1, scale=3.0), rnd(M, D, seed=2, dt=dt), rnd(D, seed=3, dt=dt)
    xd = x.to(DEV)
    xb = xd if dt == F32 else torch.empty(M, D, dtype=BF, device=DEV)
    ops.postnorm_residual_(xd, xb, y.to(DEV), w.to(DEV), 1e-4, 1.0)
    want = x.double() + V.centred_rms_norm(y.double(), w.double(), 1e-4)
    assert rel_err(xd, want) < 2e-6                               # the stream itself is fp32 in both storage types
    assert torch.equal(xb.cpu(), xd.cpu().to(dt))
    got = ops.rmsnorm_stream(xd, w.to(DEV), 1e-4, 1.0)
    assert rel_err(got, V.centred_rms_norm(xd.cpu().double(), w.double(), 1e-4)) < tol(dt)
    g = rnd(M, D + 24, seed=4, dt=dt)
    got = ops.gated_norm(y.to(DEV), g.to(DEV)[:, 16:16 + D], w.to(DEV), 1e-2)
    want = V.plain_rms_norm(y.double(), w.double(), 1e-2) * torch.sigmoid(g[:, 16:16 + D].double())
    assert rel_err(got, want) < tol(dt)
    z = rnd(M, 2 * D, seed=5, dt=dt, scale=2.0)
    assert rel_err(ops.silu_gate(z.to(DEV)), V.silu(z[:, :D].double()) * z[:, D:].double()) < tol(dt)


@pytest.mark.parametrize("M,K,N", [(1, 64, 5), (2, 192, 70), (3, 1032, 33), (4, 4096, 512), (1, 4104, 1027), (4, 8192, 64), (1, 520, 48)])
def test_closing_norm_in_the_next_layers_launch(ops, M, K, N):
    y, g, x, w = rnd(M, K, seed=1, dt=BF), rnd(K, seed=2, dt=BF), rnd(M, K, seed=3), rnd(2 * N, K, seed=4, dt=BF, scale=1.0 / math.sqrt(K))
    want = x.double() + V.centred_rms_norm(y.double(), g.double(), 1e-4)
    xin = want.to(BF).double()
    yd, gd, xd, wd = (t.to(DEV) for t in (y, g, x, w))
    out = torch.empty_like(xd)
    z = ops.postnorm_linear(yd, gd, xd, out, wd, 1e-4, 1.0)
    assert rel_err(out, want) < 2e-6 and torch.equal(xd.cpu(), x)
    assert rel_err(z, xin @ w.double().T) < 8e-3
    t = (xin @ w.double().T).to(BF).double()
    for act, fn in (("silu", V.silu), ("gelu", torch.nn.functional.gelu)):
        want_a = fn(t[:, :N]) * t[:, N:]
        assert rel_err(ops.postnorm_gate(yd, gd, xd, out, wd, False, act, 1e-4, 1.0), want_a) < 1e-2
        if N % 32 == 0:
            assert rel_err(ops.postnorm_gate(yd, gd, xd, out, ops.pack_gate_weights(wd), True, act, 1e-4, 1.0), want_a) < 1e-2
    assert rel_err(out, want) < 2e-6


@TYPES
def test_embedding(ops, dt):
    w = rnd(37, 52, dt=dt)
    ids = torch.tensor([0, 36, 5, 5])
    x, xb = ops.embed_stream(ids.to(DEV), w.to(DEV), 0.3)
    assert x.dtype == F32 and rel_err(x, w[ids].double() * 0.3) < 1e-6 and torch.equal(xb.cpu(), x.cpu().to(dt))
    for bad in (-1, 37):
        with pytest.raises(IndexError):
            ops.embed_stream(torch.tensor([3, bad]).to(DEV), w.to(DEV), 1.0)


def test_norm_eps_is_inside_the_root(ops):
    y = torch.full((2, 64), 1e-3)
    x = torch.zeros(2, 64, device=DEV)
    ops.postnorm_residual_(x, x, y.to(DEV), torch.zeros(64, device=DEV), 1e-6, 1.0)
    assert abs(float(x[0, 0]) - 1 / math.sqrt(2)) < 1e-6


# ------------------------------------------------------------------------------------------------ gated feed-forward with SiLU
@pytest.mark.parametrize("M,I,K", [(1, 256, 192), (3, 66, 64), (5, 256, 256), (9, 128, 256), (40, 320, 512), (300, 256, 128), (257, 384, 192), (300, 70, 100)])
@pytest.mark.parametrize("grouped", [False, True])
def test_silu_gated_mlp(ops, M, I, K, grouped):
    if grouped and (I % 128 or K % 64 or K < 128):
        pytest.skip("outside the grouped layout's contract")
    x, w = rnd(M, K, seed=1, dt=BF), rnd(2 * I, K, seed=2, dt=BF, scale=1.5 / math.sqrt(K))
    wd = w.to(DEV)
    got = ops.mlp_gate(x.to(DEV), None if grouped else wd, w12g=ops.pack_gate_weights(wd) if grouped else None, act="silu")
    z = (x.double() @ w.double().T).to(BF).double()               # both products are rounded before the gate
    assert rel_err(got, V.silu(z[:, :I]) * z[:, I:]) < 6e-3


@TYPES
@pytest.mark.parametrize("M,N,K,n", [(3, 70, 52, 33), (20, 512, 128, 256), (300, 512, 192, 256), (300, 512, 192, 512), (300, 512, 192, 200), (5129, 512, 128, 256)])
def test_linear_with_silu_on_the_first_columns(ops, dt, M, N, K, n):
    x, w = rnd(M, K, seed=1, dt=dt), rnd(N, K, seed=2, dt=dt, scale=2.0 / math.sqrt(K))
    got = ops.linear_act(x.to(DEV), w.to(DEV), "silu", n)
    want = x.double() @ w.double().T
    want[:, :n] = V.silu(want[:, :n])
    assert rel_err(got, want) < tol(dt, 8e-3, 5e-6)


# ------------------------------------------------------------------------------------------------ decayed linear attention
def lightning_case(ops, dt, lens, H, dk, dv, decay, states=None, seg_len=None, extra=8, seed=0):
    from evo_amd.mixer_ops import TokenBatch
    M, n = sum(lens), H * (2 * dk + dv)
    z = rnd(M, n + extra, seed=seed, dt=dt)
    past = [0 if states is None or s is None else 5 for s in (states or [None] * len(lens))]
    batch = TokenBatch.of_prompts(lens, past, DEV)
    st = torch.full((len(lens), H, dk, dv), 1e6)                  # what a reused slot may hold
    for b, p in enumerate(past):
        if p:
            st[b] = states[b]
    st = st.to(DEV)
    dec = torch.tensor(decay, dtype=F32)
    o = ops.lightning(z.to(DEV), H, dk, dv, dec.to(DEV), torch.log2(dec.double()).float().to(DEV), batch, st, seg_len=seg_len)
    at = 0
    for b, L in enumerate(lens):
        a = z[at:at + L, :n].double()
        q, k, v = a[:, :H * dk].view(L, H, dk), a[:, H * dk:2 * H * dk].view(L, H, dk), a[:, 2 * H * dk:].view(L, H, dv)
        want, S = V.decayed_linear_attention(q, k, v, decay, states[b].double() if past[b] else None)
        assert rel_err(o[at:at + L], want.reshape(L, -1)) < tol(dt, 8e-3, 2e-5), (b, L)
        assert rel_err(st[b].reshape(1, -1), S.reshape(1, -1)) < tol(dt, 3e-5, 2e-5), (b, L)
        at += L
    return o, st


SHAPES = [(2, 64, 64), (3, 24, 40), (1, 128, 128), (2, 7, 5), (1, 33, 130), (2, 128, 64), (4, 16, 100), (1, 100, 200)]


@TYPES
@pytest.mark.parametrize("H,dk,dv", SHAPES)
def test_lightning_prompts(ops, dt, H, dk, dv):
    decay = [float(a) for a in np.linspace(0.3, 0.999, H)]
    lightning_case(ops, dt, [1, 63, 64, 65, 2, 150], H, dk, dv, decay)


@pytest.mark.parametrize("H,dk,dv", [(2, 64, 64), (1, 128, 128), (3, 24, 40)])
def test_lightning_segments_and_carried_states(ops, H, dk, dv):
    """Sequences cut into segments; some go on from a state; all forms of the cut agree with the reference."""
    decay = [0.999, 0.9, 0.4][:H]
    lens = [700, 130, 64, 1, 257]
    states = [rnd(H, dk, dv, seed=9), None, rnd(H, dk, dv, seed=10), rnd(H, dk, dv, seed=11), None]
    for seg in (64, 128, 256, 1024):
        lightning_case(ops, BF, lens, H, dk, dv, decay, states=states, seg_len=seg)
    lightning_case(ops, F32, lens, H, dk, dv, decay, states=states)


def test_lightning_decays_of_zero_and_one(ops):
    for dt in (BF, F32):
        lightning_case(ops, dt, [140, 66], 3, 32, 32, [0.0, 1.0, 0.5])


def test_lightning_wide_head_takes_the_recurrent_form(ops):
    lightning_case(ops, BF, [70, 3], 1, 150, 20, [0.95])


@TYPES
@pytest.mark.parametrize("H,dk,dv", [(2, 64, 64), (1, 128, 128), (3, 24, 40), (2, 7, 5), (1, 150, 33)])
def test_lightning_decode_step(ops, dt, H, dk, dv):
    from evo_amd.mixer_ops import TokenBatch
    B, n = 5, H * (2 * dk + dv)
    decay = [float(a) for a in np.linspace(0.2, 0.99, H)]
    st = rnd(B + 2, H, dk, dv, seed=3)
    std = st.to(DEV)
    dec = torch.tensor(decay)
    for t in range(3):
        z = rnd(B, n + 8, seed=20 + t, dt=dt)
        o = ops.lightning(z.to(DEV), H, dk, dv, dec.to(DEV), torch.log2(dec).to(DEV), TokenBatch.of_decode(torch.zeros(B, dtype=torch.int64, device=DEV)), std)
        a = V.silu(z[:, :n].double())
        for b in range(B):
            q, k, v = a[b:b + 1, :H * dk].view(1, H, dk), a[b:b + 1, H * dk:2 * H * dk].view(1, H, dk), a[b:b + 1, 2 * H * dk:].view(1, H, dv)
            want, S = V.decayed_linear_attention(q, k, v, decay, st[b].double())
            st[b] = S
            assert rel_err(o[b:b + 1], want.reshape(1, -1)) < tol(dt, 6e-3, 5e-6)
            assert rel_err(std[b].reshape(1, -1), S.reshape(1, -1)) < tol(dt, 1e-5, 5e-6)
    assert torch.equal(std[B:].cpu(), st[B:])                     # rows of other slots stay


# ------------------------------------------------------------------------------------------------ latent attention: preparation
@TYPES
@pytest.mark.parametrize("H,dn,dr,R,n_rot,ring", [(3, 24, 16, 48, 16, 7), (1, 10, 6, 33, 4, 64), (17, 8, 32, 512, 32, 100)])
def test_latent_prep(ops, dt, H, dn, dr, R, n_rot, ring):
    from evo_amd.mixer_ops import MixerOps, TokenBatch
    lens, past = [5, 1, ring + 9], [0, 1234, 3]
    M, base = sum(lens), 10000.0
    batch = TokenBatch.of_prompts(lens, past, DEV)
    nq = H * (dn + dr)
    qd, w = rnd(M, nq + R + dr, seed=1, dt=dt), rnd(R, seed=2, dt=dt)
    inv = torch.tensor([base ** (-2.0 * i / n_rot) for i in range(n_rot // 2)])
    rs = MixerOps.latent_row(R, dr)
    cache = torch.full((3, ring, rs), 5.0, dtype=dt, device=DEV)
    x = qd.to(DEV)
    c, kr = ops.latent_prep(x, H, dn, dr, R, w.to(DEV), inv.to(DEV), 1e-5, batch, cache, want_kv=True)
    pos = torch.cat([torch.arange(p, p + n) for p, n in zip(past, lens)])
    q = qd[:, :nq].double().view(M, H, dn + dr)
    want_q = torch.cat([q[..., :dn], V.rotate_half(q[..., dn:], pos, base, n_rot)], -1).reshape(M, nq)
    want_c = V.plain_rms_norm(qd[:, nq:nq + R].double(), w.double(), 1e-5)
    want_k = V.rotate_half(qd[:, nq + R:].double(), pos, base, n_rot)
    t = tol(dt, 6e-3, 2e-4)                                       # (fp32 angles of positions beyond a thousand)
    assert rel_err(x[:, :nq], want_q) < t and rel_err(c, want_c) < tol(dt) and rel_err(kr, want_k) < t
    at = 0
    for b, (p, n) in enumerate(zip(past, lens)):
        seen = set()
        for i in range(max(0, n - ring), n):
            s = (p + i) % ring
            seen.add(s)
            assert torch.equal(cache[b, s, :R], c[at + i]) and torch.equal(cache[b, s, R:R + dr], kr[at + i])
            assert bool((cache[b, s, R + dr:] == 5.0).all())      # the padding of a row is never written
        assert all(bool((cache[b, s] == 5.0).all()) for s in range(ring) if s not in seen)
        at += n


# ------------------------------------------------------------------------------------------------ latent attention: prompts
def spiky_window_case(lq, lk, H, dn, dr, dv, dt, seed):
    """Random queries and keys plus keys that stand out for every query: an edge off by one moves the output by its full size."""
    q, kn, kr = rnd(lq, H, dn + dr, seed=seed), rnd(lk, H, dn, seed=seed + 1), rnd(lk, dr, seed=seed + 2)
    v = rnd(lk, H, dv, seed=seed + 3)
    q[..., 0] = 3.0
    for j in range(0, lk, 23):
        kn[j, :, 0] += 14.0
    return [t.to(dt) for t in (q, kn, kr, v)]


@TYPES
@pytest.mark.parametrize("H,dn,dr,dv,window", [
    (2, 32, 32, 64, 41), (3, 24, 16, 40, 1), (1, 64, 32, 128, 64), (2, 64, 64, 80, 65), (1, 128, 64, 128, 63), (2, 10, 6, 9, 17), (1, 160, 64, 32, 129),
    (1, 100, 20, 200, 128), (2, 8, 8, 16, 10 ** 6), (1, 200, 100, 300, 33)])
def test_window_attention(ops, mfma, dt, H, dn, dr, dv, window):
    if not mfma and dt == F32:
        pytest.skip("fp32 has the any-size kernel only")
    lens = [1, 2, 64, 65, 200, 129, 16]
    extra = [0, 3, 5, 0, min(window - 1, 70), 0, 1]               # earlier keys a sequence still sees
    sink = rnd(H, seed=7, scale=2.0)
    parts = [spiky_window_case(n, n + e, H, dn, dr, dv, dt, 100 * i) for i, (n, e) in enumerate(zip(lens, extra))]
    pad = 8 if dn % 8 == 0 and dr % 8 == 0 else 3
    qd = torch.cat([torch.cat([p[0].reshape(len(p[0]), -1), torch.zeros(len(p[0]), pad, dtype=dt)], 1) for p in parts])
    kv = torch.cat([torch.cat([p[1].reshape(len(p[1]), -1), p[3].reshape(len(p[3]), -1)], 1) for p in parts])
    kr = torch.cat([p[2] for p in parts])
    cu = lambda ns: torch.tensor([0] + ns).cumsum(0).to(torch.int32).to(DEV)
    scale = 1.0 / math.sqrt(dn + dr)
    got = ops.window_attention(qd.to(DEV), kv.to(DEV), kr.to(DEV), H, dn, dr, dv, window, scale, sink.to(DEV), cu(lens),
                               cu([n + e for n, e in zip(lens, extra)]), max(lens))
    at = 0
    for (q, kn, kr_, v), n, e in zip(parts, lens, extra):
        k = torch.cat([kn, kr_[:, None].expand(n + e, H, dr)], -1).double()
        pos = torch.arange(n + e)
        want = V.windowed_sink_attention(q.double(), k, v.double(), scale, window, sink, pos[e:], pos).reshape(n, -1)
        assert rel_err(got[at:at + n], want) < tol(dt, 1.2e-2, 1e-5), (n, e)
        at += n


def test_latent_split_covers_the_window():
    from evo_amd.mixer_ops import MixerOps
    for B in (1, 3, 8, 33, 300):
        for heads in (1, 16, 17, 128):
            for tiles in (1, 5, 64, 1000):
                n, group = MixerOps.latent_split(B, heads, tiles)
                assert 1 <= n <= min(tiles, 64) and group in (16, 32)


def test_sink_takes_its_share(ops, mfma):
    """All scores zero: a window of n keys and a sink of log(n) give half the mean value."""
    T, W = 100, 20
    qd, kv, kr = torch.zeros(T, 16, dtype=BF), torch.zeros(T, 16, dtype=BF), torch.zeros(T, 8, dtype=BF)
    kv[:, 8:] = 1.0
    cu = torch.tensor([0, T], dtype=torch.int32, device=DEV)
    got = ops.window_attention(qd.to(DEV), kv.to(DEV), kr.to(DEV), 1, 8, 8, 8, W, 1.0, torch.tensor([math.log(W)]).to(DEV), cu, cu, T).float().cpu()
    n = torch.arange(1, T + 1).clamp(max=W)
    assert torch.allclose(got[:, 0], n / (n + W), atol=4e-3)


# ------------------------------------------------------------------------------------------------ latent attention: decode
@TYPES
@pytest.mark.parametrize("H,dn,dr,dv,R,window,ring", [
    (3, 24, 16, 40, 48, 9, 9), (5, 32, 16, 72, 128, 45, 45), (1, 10, 6, 9, 33, 17, 20), (17, 64, 32, 64, 160, 64, 64), (2, 128, 64, 128, 512, 100, 100),
    (16, 16, 8, 24, 300, 33, 64), (4, 64, 0, 64, 96, 1, 1), (2, 24, 24, 17, 600, 70, 70), (33, 16, 32, 16, 64, 300, 300)])
def test_latent_decode(ops, mfma, dt, H, dn, dr, dv, R, window, ring):
    from evo_amd.mixer_ops import MixerOps
    if not mfma and dt == F32:
        pytest.skip("fp32 has the any-size kernel only")
    rs = MixerOps.latent_row(R, dr)
    pos = [0, window - 1, window, ring + 5, 3 * ring + window // 2]
    B = len(pos)
    cache = torch.full((B + 1, ring, rs), 30.0)                   # a slot outside the window must not be seen, whatever it holds
    lat = [rnd(p + 1, R + dr, seed=50 + b) for b, p in enumerate(pos)]
    for b, p in enumerate(pos):
        cache[b, :, R + dr:] = 0.0
        for j in range(0, p + 1, 13):
            lat[b][j] *= 2.5
        for j in range(max(0, p + 1 - ring), p + 1):
            cache[b, j % ring, :R + dr] = lat[b][j]
    q = rnd(B, H * (dn + dr) + 8, seed=1, dt=dt)
    wuk, wuv = rnd(H * dn, R, seed=2, dt=dt, scale=1.5 / math.sqrt(R)), rnd(H * dv, R, seed=3, dt=dt, scale=1 / math.sqrt(R))
    sink, scale = rnd(H, seed=4), 1.5 / math.sqrt(dn + dr)
    cache = cache.to(dt)
    for n_split in (None, 1, 3):
        got = ops.latent_decode(q.to(DEV), cache.to(DEV), torch.tensor(pos).to(DEV), wuk.to(DEV), wuv.to(DEV), sink.to(DEV), H, dn, dr, dv, R, window,
                                scale, n_split=n_split)
        for b, p in enumerate(pos):
            js = range(max(0, p - window + 1), p + 1)
            rows = torch.stack([cache[b, j % ring, :R + dr] for j in js]).double()
            k = torch.cat([(rows[:, :R] @ wuk.double().T).view(len(js), H, dn), rows[:, None, R:].expand(len(js), H, dr)], -1)
            v = (rows[:, :R] @ wuv.double().T).view(len(js), H, dv)
            want = V.windowed_sink_attention(q[b:b + 1, :H * (dn + dr)].double().view(1, H, dn + dr), k, v, scale, window, sink, torch.tensor([p]),
                                             torch.tensor(list(js)))
            assert rel_err(got[b:b + 1], want.reshape(1, -1)) < tol(dt, 2e-2, 1e-5), (b, p, n_split)
