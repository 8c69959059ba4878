"""GPU: the gated linear recurrence, the norm of the sum and the activations against the plain fp64 functions of oracle/batodra_ref.py, in both storage
types, at sizes around the tiles' edges."""
import math

import pytest
import torch

from oracle import batodra_ref as R
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


def rnd(*shape, seed=0, dt=F32, scale=1.0):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(*shape, generator=g) * scale).to(dt)


def tol(dt, bf=6e-3, f=5e-6):
    return bf if dt == BF else f


# ------------------------------------------------------------------------------------------------ recurrence
def layer(W, nb, taps, dt, seed=0):
    bs = W // nb
    return dict(conv=rnd(W, taps, seed=seed + 1, dt=dt, scale=0.6), conv_b=rnd(W, seed=seed + 2, dt=dt, scale=0.3), ra=rnd(nb, bs, bs, seed=seed + 3, dt=dt, scale=1.5 / math.sqrt(bs)),
                ra_b=rnd(nb, bs, seed=seed + 4, dt=dt), ri=rnd(nb, bs, bs, seed=seed + 5, dt=dt, scale=1.5 / math.sqrt(bs)), ri_b=rnd(nb, bs, seed=seed + 6, dt=dt),
                lam=rnd(W, seed=seed + 7, dt=dt, scale=1.5) - 3.0)


def decay_of(w):
    return (-8.0 * torch.nn.functional.softplus(w["lam"].double())).float()


def run_kernel(ops, z, in_b, act, W, w, batch, state, **kw):
    g = {k: t.to(DEV) for k, t in w.items()}
    return ops.rglru(z.to(DEV), None if in_b is None else in_b.to(DEV), act, W, g["conv"], g["conv_b"], g["ra"], g["ra_b"], g["ri"], g["ri_b"], decay_of(w).to(DEV), batch, state, **kw)


def plain(x, y, w, before, S):
    """-> (o, last inputs, S); the matrix-core kernels keep the convolution's result in the storage type"""
    from evo_amd.mixer_ops import MixerOps
    u, tail = R.causal_convolution(x, w["conv"].double(), w["conv_b"].double(), before)
    if MixerOps.rglru_mfma_ok(w["conv"].shape[0], w["ra"].shape[0], w["conv"].shape[1], w["ra"].dtype):
        u = u.to(BF).double()
    r, i = (torch.sigmoid(R.block_diagonal(u, w[m].double(), w[m + "_b"].double())) for m in ("ra", "ri"))
    s, last = R.gated_linear_recurrence(u, r, i, w["lam"].double(), S)
    return s * y, tail, last


def prompt_case(ops, dt, lens, W, nb, taps, past=None, seg_len=None, seed=0):
    from evo_amd.mixer_ops import TokenBatch
    M, w = sum(lens), layer(W, nb, taps, dt, seed)
    past = past or [0] * len(lens)
    z = rnd(M, 2 * W + 8, seed=seed + 20, dt=dt)
    batch = TokenBatch.of_prompts(lens, past, DEV)
    state = torch.full((len(lens) + 1, 1 + taps, W), 1e6)          # what a reused row may hold
    carried = []
    for b, p in enumerate(past):
        if not p:
            carried.append((None, None))
            continue
        S, h = rnd(W, seed=seed + 30 + b).double(), rnd(taps, W, seed=seed + 40 + b, dt=dt)
        state[b, 0] = S
        before = torch.zeros(taps - 1, W, dtype=torch.float64)
        for k in range(1, taps):
            if p - k >= 0:
                state[b, 1 + (p - k) % taps] = h[k]
                before[taps - 1 - k] = h[k].double()
        carried.append((before, S.float().double()))
    st = state.to(DEV)
    o = run_kernel(ops, z, None, False, W, w, batch, st, seg_len=seg_len)
    at = 0
    for b, L in enumerate(lens):
        y, x = z[at:at + L, :W].double(), z[at:at + L, W:2 * W].double()
        want, tail, last = plain(x, y, w, *carried[b])
        assert rel_err(o[at:at + L], want) < tol(dt, 1e-2, 3e-5), (b, L)
        assert rel_err(st[b, :1], last[None]) < tol(dt, 2e-3, 3e-5), (b, L)
        for k in range(1, taps):                                  # the convolution's last inputs, at their positions
            p = past[b] + L - k
            if p >= 0:
                assert torch.equal(st[b, 1 + p % taps].cpu().double(), tail[taps - 1 - k])
        at += L
    assert torch.equal(st[len(lens)].cpu(), state[len(lens)])


SIZES = [(96, 4, 4), (64, 1, 4), (352, 4, 3), (54, 3, 5), (320, 2, 2), (512, 2, 3), (128, 1, 1), (768, 2, 4), (272, 2, 4), (800, 2, 4), (24, 3, 4), (30, 2, 3)]


@TYPES
@pytest.mark.parametrize("W,nb,taps", SIZES)
def test_recurrence_of_prompts(ops, dt, W, nb, taps):
    prompt_case(ops, dt, [1, 63, 64, 65, 2, 150, 3], W, nb, taps)


@TYPES
@pytest.mark.parametrize("W,nb,taps", [(96, 4, 4), (320, 2, 2), (54, 3, 5), (512, 2, 3), (800, 2, 4)])
def test_recurrence_goes_on(ops, dt, W, nb, taps):
    """Carried states and convolution inputs; portions shorter than the convolution; sequences younger than it."""
    prompt_case(ops, dt, [2, 1, 70, 64, 5, 2, 130], W, nb, taps, past=[1, 2, 0, 77, 1000, 3, 64], seed=5)


@pytest.mark.parametrize("W,nb,taps", [(96, 4, 4), (352, 4, 3), (512, 2, 3), (800, 2, 4)])
@pytest.mark.parametrize("seg", [64, 128, 320, 1024])
def test_recurrence_in_segments(ops, W, nb, taps, seg):
    prompt_case(ops, BF, [700, 130, 64, 1, 321], W, nb, taps, past=[9, 0, 2, 40, 0], seg_len=seg, seed=9)


def test_slow_decays_carry_far(ops):
    """A decay close to one: what the first tokens leave behind is still there 1,500 tokens later."""
    from evo_amd.mixer_ops import TokenBatch
    W, T = 64, 1500
    for dt in (BF, F32):
        w = layer(W, 1, 4, dt)
        w["lam"], w["conv_b"] = torch.full((W,), -9.5).to(dt), torch.zeros(W, dtype=dt)
        z = rnd(T, 2 * W, seed=3, dt=dt, scale=0.1)
        z[:4, W:] = 60.0
        st = torch.zeros(1, 5, W, device=DEV)
        for seg in ((None, 256) if dt == BF else (None,)):
            o = run_kernel(ops, z, None, False, W, w, TokenBatch.of_prompts([T], [0], DEV), st, seg_len=seg)
            want, _, last = plain(z[:, W:].double(), z[:, :W].double(), w, None, None)
            short, _, _ = plain(z[100:, W:].double(), z[100:, :W].double(), w, None, None)
            assert float((want[-1] - short[-1]).abs().mean()) > 0.3 * float(want[-1].abs().mean())   # the test's own point
            assert rel_err(o, want) < tol(dt, 1e-2, 5e-5) and rel_err(st[:, 0], last[None]) < tol(dt, 3e-3, 5e-5)


@TYPES
@pytest.mark.parametrize("W,nb,taps", SIZES)
@pytest.mark.parametrize("B", [1, 5, 16, 19, 40])
def test_recurrence_step(ops, dt, W, nb, taps, B):
    """Tokens one by one from a sequence's start: bias and activation in the kernel, rows at different positions, other rows untouched."""
    from evo_amd.mixer_ops import TokenBatch
    if B > 5 and W > 352:
        pytest.skip("covered at fewer rows")
    w, in_b = layer(W, nb, taps, dt, 3), rnd(2 * W + 8, seed=77, dt=dt)
    state = rnd(B + 2, 1 + taps, W, seed=3)
    pos = [int(p) for p in torch.randint(0, 9, (B,), generator=torch.Generator().manual_seed(B))]
    before, S = [], []
    for b, p in enumerate(pos):
        h = torch.zeros(taps - 1, W, dtype=torch.float64)
        for k in range(1, taps):
            if p - k >= 0:
                h[taps - 1 - k] = state[b, 1 + (p - k) % taps].double()
        before.append(h)
        S.append(state[b, 0].double())
    std = state.to(DEV)
    for t in range(6):
        z = rnd(B, 2 * W + 8, seed=20 + t, dt=dt)
        o = run_kernel(ops, z, in_b, True, W, w, TokenBatch.of_decode((torch.tensor(pos) + t).to(DEV)), std)
        yx = z[:, :2 * W].double() + in_b[:2 * W].double()
        for b in range(B):
            want, before[b], S[b] = plain(yx[b:b + 1, W:], R.gelu_tanh(yx[b:b + 1, :W]), w, before[b], S[b])
            assert rel_err(o[b:b + 1], want) < tol(dt, 1.2e-2, 1e-5), (b, t)
            assert rel_err(std[b, :1], S[b][None]) < tol(dt, 4e-3, 1e-5), (b, t)
            S[b] = std[b, 0].cpu().double()
    assert torch.equal(std[B:].cpu(), state[B:])


# ------------------------------------------------------------------------------------------------ norm of the sum, activations
@TYPES
@pytest.mark.parametrize("M,D", [(1, 8), (3, 100), (5, 192), (70, 4096), (2, 4104), (2, 5001), (33, 1032)])
@pytest.mark.parametrize("offset", [0.0, 1.0])
def test_norm_of_the_sum(ops, dt, M, D, offset):
    x, y, w = rnd(M, D, seed=1, scale=3.0), rnd(M, D, seed=2, dt=dt, scale=2.0), rnd(D, seed=3, dt=dt)
    xd = x.to(DEV)
    xb = xd if dt == F32 else torch.empty(M, D, dtype=BF, device=DEV)
    ops.sum_norm_(xd, xb, y.to(DEV), w.to(DEV), 0.6, 1e-2, offset)
    assert rel_err(xd, R.norm_of_sum(x.double(), y.double(), 0.6, offset + w.double(), 1e-2)) < 2e-6
    assert torch.equal(xb.cpu(), xd.cpu().to(dt))


@pytest.mark.parametrize("M,K,N", [(1, 64, 5), (2, 192, 70), (3, 1032, 33), (4, 4096, 512), (1, 4104, 1027), (4, 8192, 64), (1, 520, 48)])
def test_norm_of_the_sum_in_the_next_layers_launch(ops, M, K, N):
    y, g, x, w = rnd(M, K, seed=1, dt=BF), rnd(K, seed=2, dt=BF), rnd(M, K, seed=3), rnd(2 * N, K, seed=4, dt=BF, scale=1.0 / math.sqrt(K))
    want = R.norm_of_sum(x.double(), y.double(), 2.5, g.double(), 1e-4)
    xin = want.to(BF).double()
    yd, gd, xd, wd = (t.to(DEV) for t in (y, g, x, w))
    out = torch.empty_like(xd)
    z = ops.postnorm_linear(yd, gd, xd, out, wd, 1e-4, 0.0, alpha=2.5)
    assert rel_err(out, want) < 2e-6 and torch.equal(xd.cpu(), x)
    plain_z = xin @ w.double().T
    assert rel_err(z, plain_z) < 8e-3
    assert rel_err(ops.postnorm_linear(yd, gd, xd, out, wd, 1e-4, 0.0, alpha=2.5, act="relu2"), R.squared_relu(plain_z)) < 1e-2
    assert rel_err(ops.postnorm_linear(yd, gd, xd, out, wd, 1e-4, 0.0, alpha=2.5, act="gelu_tanh"), R.gelu_tanh(plain_z)) < 1e-2
    t = plain_z.to(BF).double()
    assert rel_err(ops.postnorm_gate(yd, gd, xd, out, wd, False, "silu", 1e-4, 0.0, alpha=2.5), V.silu(t[:, :N]) * t[:, N:]) < 1e-2
    before = x.double() + V.centred_rms_norm(y.double(), g.double(), 1e-4)          # the other order, with the activation
    got = ops.postnorm_linear(yd, gd, xd, out, wd, 1e-4, 1.0, act="relu2")
    assert rel_err(out, before) < 2e-6 and rel_err(got, R.squared_relu(before.to(BF).double() @ w.double().T)) < 1e-2


@TYPES
@pytest.mark.parametrize("act,fn", [("silu", V.silu), ("gelu_tanh", R.gelu_tanh), ("relu2", R.squared_relu)])
@pytest.mark.parametrize("bias", [False, True])
@pytest.mark.parametrize("M,N,K,n", [(3, 70, 52, 33), (20, 512, 128, 256), (300, 512, 192, 256), (300, 512, 192, 512), (300, 512, 192, 200), (5129, 512, 128, 256), (40, 1280, 256, 1280),
                                     (1, 70, 64, 70), (4, 4096, 2048, 4096), (7, 128, 72, 128), (9, 8192, 256, 8192), (33, 8192, 256, 8192), (33, 2048, 8192, 2048), (64, 320, 96, 320)])
def test_linear_with_activation(ops, dt, act, fn, bias, M, N, K, n):
    x, w, b = rnd(M, K, seed=1, dt=dt), rnd(N, K, seed=2, dt=dt, scale=2.0 / math.sqrt(K)), rnd(N, seed=3, dt=dt)
    got = ops.linear_act(x.to(DEV), w.to(DEV), act, n, b.to(DEV) if bias else None)
    want = x.double() @ w.double().T + (b.double() if bias else 0.0)
    want[:, :n] = fn(want[:, :n])
    assert rel_err(got, want) < tol(dt, 9e-3, 5e-6)


def test_activations_far_out(ops):
    z = torch.tensor([[-1e4, -50.0, -5.0, -0.0, 0.0, 1e-3, 5.0, 50.0, 1e4, 3e38, -3e38]])
    for dt in (BF, F32):
        for act, fn in (("gelu_tanh", R.gelu_tanh), ("silu", V.silu), ("relu2", R.squared_relu)):
            x = z.to(dt).to(DEV)
            ops.act_cols_(x, 9, act)
            want = fn(z.to(dt).double())[:, :9]
            assert torch.allclose(x[:, :9].cpu().double(), want, rtol=1e-2 if dt == BF else 1e-5, atol=2e-4) and torch.equal(x[:, 9:].cpu(), z.to(dt)[:, 9:])
