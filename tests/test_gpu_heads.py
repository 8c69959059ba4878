"""GPU: attention with cached keys and values -- preparation, prompts, decode -- against the plain fp64 functions of oracle/batodra_ref.py, in both
storage types, at sizes around the tiles' edges."""
import math

import pytest
import torch

from oracle import batodra_ref as R
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


# ------------------------------------------------------------------------------------------------ preparation
@TYPES
@pytest.mark.parametrize("nq,nk,dim,nv,n_rot,keep,window", [
    (4, 2, 128, 96, 128, 3, 9), (6, 2, 48, 40, 16, 0, 64), (3, 1, 10, 9, 6, 2, 5), (2, 2, 64, 64, 0, 5, 1), (8, 4, 32, 24, 32, 0, 500), (1, 1, 24, 8, 16, 1, 3),
    (2, 1, 40, 16, 32, 4, 7), (3, 3, 8, 8, 8, 0, 2), (2, 1, 256, 256, 64, 0, 30), (70, 1, 16, 16, 16, 2, 30)])
@pytest.mark.parametrize("norm", ["weights", "unit", "both", "none"])
def test_heads_prep(ops, dt, nq, nk, dim, nv, n_rot, keep, window, norm):
    from evo_amd.mixer_ops import TokenBatch
    lens, past = [5, 1, window + 9], [0, 1234, 3]
    M, base, amp, eps = sum(lens), 10000.0, 1.3, 1e-3
    batch = TokenBatch.of_prompts(lens, past, DEV)
    cols = (nq + nk) * dim + nv
    z = rnd(M, (cols + 15) // 8 * 8, seed=1, dt=dt)
    qw, kw = (rnd(dim, seed=s, dt=dt) for s in (2, 3))
    freqs = R.rotation_frequencies(base, n_rot) if n_rot else []
    rs = (nk * dim + nv + 7) // 8 * 8
    cache = torch.full((3, keep + window, rs), 5.0, dtype=dt, device=DEV)
    x = z.to(DEV)
    weights, unit = norm in ("weights", "both"), norm in ("unit", "both")
    ops.heads_prep(x, nq, nk, dim, nv, (qw.to(DEV), kw.to(DEV)) if weights else None, torch.tensor(freqs, dtype=torch.float64).float().to(DEV), amp, unit, eps,
                   batch, cache, keep)
    pos = torch.cat([torch.arange(p, p + n) for p, n in zip(past, lens)])
    v = z[:, :(nq + nk) * dim].double().view(M, nq + nk, dim)
    if weights:
        v = torch.cat([R.rms_norm(v[:, :nq], qw.double(), eps), R.rms_norm(v[:, nq:], kw.double(), eps)], 1)
    v = R.rotate(v, pos, freqs, amp)
    v = R.unit_rms(v, eps) if unit else v
    assert rel_err(x[:, :(nq + nk) * dim], v.reshape(M, -1)) < tol(dt, 6e-3, 2e-4)         # (fp32 angles of positions beyond a thousand)
    assert torch.equal(x[:, (nq + nk) * dim:].cpu(), z[:, (nq + nk) * dim:])
    at = 0
    for b, (p, n) in enumerate(zip(past, lens)):
        seen = set()
        for i in range(n):
            if p + i >= keep and n - i > window:
                continue
            s = p + i if p + i < keep else keep + (p + i - keep) % window
            seen.add(s)
            assert torch.equal(cache[b, s, :nk * dim + nv], x[at + i, nq * dim:cols])
        assert all(bool((cache[b, s] == 5.0).all()) for s in range(keep + window) if s not in seen)
        at += n


# ------------------------------------------------------------------------------------------------ prompts
def combine(q, k, v, maps, scale, lam, gain, eps, mask):
    if maps == 1:
        return R.softmax_attention(q, k, v, scale, mask)
    a1, a2 = (R.softmax_attention(q[:, i::2], k[:, i::2], v, scale, mask) for i in (0, 1))
    return gain * R.unit_rms(a1 - lam * a2, eps)


def spiky(lq, lk, H, G, maps, n, dv, dt, seed):
    """Random queries and keys plus keys that stand out for every query: an edge off by one moves the output by its full size."""
    q, k, v = rnd(lq, H * maps, n, seed=seed), rnd(lk, G * maps, n, seed=seed + 1), rnd(lk, G, dv, seed=seed + 2)
    q[..., 0] = 3.0
    for j in range(0, lk, 23):
        k[j, ::2, 0] += 14.0                                      # (every head; of two maps the first)
    return [t.to(dt) for t in (q, k, v)]


CASES = [(2, 2, 1, 32, 64, 41, 5), (6, 2, 1, 56, 40, 120, 6), (3, 1, 1, 10, 9, 17, 3), (4, 1, 1, 64, 128, 64, 70), (1, 1, 1, 128, 128, 65, 1), (2, 2, 1, 160, 40, 33, 64),
         (2, 1, 1, 192, 128, 63, 2), (1, 1, 1, 256, 256, 100, 9), (8, 2, 1, 16, 24, 1, 1), (2, 2, 1, 300, 300, 33, 7), (2, 2, 1, 24, 200, None, 0), (3, 3, 2, 56, 112, None, 0),
         (4, 2, 2, 64, 64, None, 0), (2, 1, 2, 128, 256, None, 0), (3, 1, 2, 7, 11, None, 0), (2, 2, 2, 96, 128, 50, 6), (1, 1, 2, 16, 160, 64, 0), (2, 2, 2, 150, 20, None, 0),
         (2, 1, 2, 24, 256, 33, 130), (5, 5, 2, 40, 30, None, 0), (2, 1, 2, 128, 256, 70, 3)]


@TYPES
@pytest.mark.parametrize("H,G,maps,n,dv,window,keep", CASES)
def test_prompt_attention(ops, mfma, dt, H, G, maps, n, dv, window, keep):
    if not mfma and dt == F32:
        pytest.skip("fp32 has the any-size kernel only")
    lens = [1, 2, 64, 65, 200, 129, 300]
    extra = [0, 3, 5, 0, 70 if window is None else min(window - 1, 70), 0, 1]      # earlier keys a sequence still sees
    parts = [spiky(m, m + e, H, G, maps, n, dv, dt, 100 * i) for i, (m, e) in enumerate(zip(lens, extra))]
    z = torch.cat([torch.cat([p[0].reshape(len(p[0]), -1), torch.zeros(len(p[0]), 8, dtype=dt)], 1) for p in parts])
    kv = torch.cat([torch.cat([p[1].reshape(len(p[1]), -1), p[2].reshape(len(p[2]), -1)], 1) for p in parts])
    cu = lambda ns: torch.tensor([0] + ns).cumsum(0).to(torch.int32).to(DEV)
    scale, lam, gain, eps = 1.0 / math.sqrt(n), 0.45, 0.7, 1e-4
    got = ops.heads_attention(z.to(DEV), kv.to(DEV), H, G, maps, n, dv, window, keep, scale, lam, gain, eps, cu(lens), cu([m + e for m, e in zip(lens, extra)]), max(lens))
    at = 0
    for (q, k, v), m, e in zip(parts, lens, extra):
        pos = torch.arange(m + e)
        want = combine(q.double(), k.double(), v.double(), maps, scale, lam, gain, eps, R.visible(pos[e:], pos, window, keep)).reshape(m, -1)
        assert rel_err(got[at:at + m], want) < tol(dt, 1.5e-2 if maps == 1 else 2.5e-2, 2e-5), (m, e)
        at += m


def test_query_that_sees_one_token_only(ops, mfma):
    """A window of one token without kept ones: the output is the token's own value, whatever the scores."""
    T, n, dv = 130, 32, 64
    q, k, v = rnd(T, 2, n, seed=1, dt=BF, scale=9.0), rnd(T, 1, n, seed=2, dt=BF, scale=9.0), rnd(T, 1, dv, seed=3, dt=BF)
    cu = torch.tensor([0, T], dtype=torch.int32, device=DEV)
    got = ops.heads_attention(q.reshape(T, -1).to(DEV), torch.cat([k[:, 0], v[:, 0]], 1).to(DEV), 2, 1, 1, n, dv, 1, 0, 1.0, 0.0, 1.0, 0.0, cu, cu, T)
    assert torch.equal(got.cpu().view(T, 2, dv), v.expand(T, 2, dv))


# ------------------------------------------------------------------------------------------------ decode
@TYPES
@pytest.mark.parametrize("H,G,maps,n,dv,keep,window", [
    (2, 2, 1, 32, 64, 3, 9), (6, 2, 1, 56, 40, 6, 120), (3, 1, 1, 10, 9, 1, 20), (40, 2, 1, 64, 128, 0, 64), (4, 4, 1, 128, 128, 2, 300), (2, 1, 1, 256, 256, 0, 33),
    (2, 2, 1, 300, 300, 5, 40), (4, 1, 1, 96, 200, 0, 1), (3, 3, 2, 56, 112, 0, 700), (17, 1, 2, 64, 64, 0, 200), (2, 1, 2, 128, 256, 0, 130), (3, 1, 2, 7, 11, 0, 50),
    (2, 2, 2, 24, 40, 7, 65), (2, 2, 2, 150, 20, 0, 70)])
def test_decode_attention(ops, mfma, dt, H, G, maps, n, dv, keep, window):
    if not mfma and dt == F32:
        pytest.skip("fp32 has the any-size kernel only")
    ring = keep + window
    rs = (G * (maps * n + dv) + 7) // 8 * 8
    pos = [0, 1, ring - 1, ring, 3 * ring + window // 2, min(31, ring), 63]
    B = len(pos)
    cache = torch.zeros(B + 1, ring, rs)
    kept = []                                                     # the visible tokens of every sequence
    for b, p in enumerate(pos):
        k, v = rnd(p + 1, G * maps, n, seed=50 + b), rnd(p + 1, G, dv, seed=90 + b)
        for j in range(0, p + 1, 13):
            k[j, ::2, 0] += 6.0
        cache[b, :, :] = 0.0
        for j in range(p + 1):
            if j < keep or p - j < window:
                cache[b, j if j < keep else keep + (j - keep) % window, :G * (maps * n + dv)] = torch.cat([k[j].reshape(-1), v[j].reshape(-1)])
        at = torch.tensor([j for j in range(p + 1) if j < keep or p - j < window])
        kept.append((k[at].to(dt), v[at].to(dt)))
    z = rnd(B, H * maps * n + 8 - H * maps * n % 8, seed=1, dt=dt)
    z[:, :H * maps * n:n] = 3.0
    scale, lam, gain, eps = 1.0 / math.sqrt(n), 0.45, 0.7, 1e-4
    cache = cache.to(dt)
    for n_split in (None, 1, 3):
        got = ops.heads_decode(z.to(DEV), cache.to(DEV), torch.tensor(pos).to(DEV), H, G, maps, n, dv, scale, lam, gain, eps, n_split=n_split)
        for b in range(B):
            k, v = (t.double() for t in kept[b])
            want = combine(z[b:b + 1, :H * maps * n].double().view(1, H * maps, n), k, v, maps, scale, lam, gain, eps, torch.ones(1, len(k), dtype=torch.bool))
            assert rel_err(got[b:b + 1], want.reshape(1, -1)) < tol(dt, 1.5e-2 if maps == 1 else 3e-2, 2e-5), (b, n_split)


def test_split_covers_the_cache():
    from evo_amd.mixer_ops import MixerOps
    for groups in (1, 8, 300, 5000):
        for ring in (1, 128, 129, 5000, 1 << 20):
            n = MixerOps.heads_split(groups, ring)
            assert 1 <= n <= max(1, (ring + 127) // 128) and n <= 64
