"""Prefill and decode throughput of a Vozalorn or Batodra model at the layer sizes of a 7B model (random weights), beside the framework's closest
models of the same width, depth and feed-forward weights, through prompt passes and pooled decode steps; per-kernel times with the fraction of
the part's peak each reaches.  Run as `python bench.py --arch vozalorn` or `--arch batodra`."""
import json
import math
import sys
import time

import torch

HBM = 8.0e12
MFMA = 2.5e15
WIDTH, FF, HEADS = 4096, 11008, 32
LATENT = dict(heads=HEADS, dim=128, rot_dim=64, vdim=128, kv_rank=512, window=1024)
LIGHT = dict(heads=HEADS, dim=128, vdim=128)
PLAIN_FF = 16384                 # two matrices with as many weights as three of FF
WINDOWED = dict(heads=32, kv_heads=8, dim=128, vdim=128, mask=dict(size=1024, keep_first=4))
DIFFERENTIAL = dict(heads=16, kv_heads=16, dim=128, vdim=256)
RGLRU = dict(width=4096, blocks=16, conv=4)
BESIDE = {"vozalorn": ["stripedhyena"], "batodra": ["vozalorn", "stripedhyena"]}


def vozalorn_config(n_layers):
    l = LATENT
    lat = dict(type="latent_attention", mlp=dict(kind="dense", ff=FF),
               mixer=dict(heads=l["heads"], dim=l["dim"], rot_dim=l["rot_dim"], vdim=l["vdim"], kv_rank=l["kv_rank"], mask=dict(size=l["window"]),
                          rot=dict(base=10000.0, dims=l["rot_dim"]), scale=(l["dim"] + l["rot_dim"]) ** -0.5))
    lin = dict(type="lightning", mlp=dict(kind="dense", ff=FF), mixer=dict(decay=[1 - 2.0 ** (-1 - 9 * h / HEADS) for h in range(HEADS)], **LIGHT))
    return dict(architecture="Vozalorn", vocab=512, width=WIDTH, norm=dict(eps=1e-6), embedding=dict(scale=1.0),
                layers=[lin if i % 2 else lat for i in range(n_layers)])


def batodra_config(n_layers):
    ff = dict(kind="dense", ff=PLAIN_FF)
    rot = dict(base=10000.0, dims=128)
    win = dict(type="attention_2", mlp=ff, mixer=dict(scale=128 ** -0.5, rot=dict(rot, scaling=dict(factor=4.0, original=4096, fast=32.0, slow=1.0)), **WINDOWED))
    dif = dict(type="attention", mlp=ff, mixer=dict(scale=128 ** -0.5, diff=0.5, rot=rot, **DIFFERENTIAL))
    rec = dict(type="rglru", mlp=ff, mixer=RGLRU)
    return dict(architecture="Batodra", vocab=512, width=WIDTH, norm=dict(eps=1e-6), postln_alpha=2.0, layers=[(win, rec, dif, rec)[i % 4] for i in range(n_layers)])


def hyena_config(n_layers):
    return dict(vocab_size=512, hidden_size=WIDTH, num_layers=n_layers, attn_layer_idxs=list(range(1, n_layers, 2)), num_attention_heads=HEADS,
                inner_mlp_size=FF)


def build(kind, n_layers, device):
    from evo_amd.models import architecture_of
    from evo_amd.synthetic import synthetic_state_dict
    config = {"vozalorn": vozalorn_config, "batodra": batodra_config, "stripedhyena": hyena_config}[kind](n_layers)
    m = architecture_of(config)(config)
    m.load_state_dict(synthetic_state_dict(m, seed=0, device=device), strict=True)
    if kind == "stripedhyena":
        m.to_bfloat16_except_poles_residues()
    m = m.to(device)
    if kind == "stripedhyena":
        m.prepare()
    return m


def progress(line):
    print(line, file=sys.stderr, flush=True)


def weight_bytes(m):
    return sum(t.numel() * t.element_size() for k, t in m.state_dict().items() if k not in ("embed", "embedding_layer.weight"))


def seconds(fn, steps, warmup=2):
    for _ in range(warmup):
        fn()
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(steps):
        fn()
    torch.cuda.synchronize()
    return (time.perf_counter() - t0) / steps


def kernel_times(m, fn):
    from evo_amd.ops import KernelTimer
    fn()
    torch.cuda.synchronize()
    m.ops.timer = KernelTimer()
    try:
        for _ in range(3):
            fn()
        torch.cuda.synchronize()
        return {k: [n // 3, ms * 1e3] for k, (n, ms) in m.ops.timer.summary().items()}
    finally:
        m.ops.timer = None


def prefill_work(B, T):
    """{kernel: (bytes, flop)} of one launch over B prompts of T tokens"""
    M, D, H = B * T, WIDTH, HEADS
    l, W = LATENT, min(LATENT["window"], T)
    pairs = B * H * (W * (W + 1) // 2 + (T - W) * W)
    n = H * (l["dim"] + l["rot_dim"]) + l["kv_rank"] + l["rot_dim"]
    return {"postnorm_residual": (12 * M * D, 0), "gated_norm": (6 * M * D, 0),
            "lightning_chunk_bf16": (8 * M * D, M * H * 128 * 128 * 2 * 3),
            "window_attn": (0, 2 * pairs * (l["dim"] + l["rot_dim"] + l["vdim"])), "attn_fwd": (0, 2 * B * H * (T * (T + 1) // 2) * 256),
            "latent_prep": (M * 2 * (n + H * l["rot_dim"] + 2 * (l["kv_rank"] + l["rot_dim"])), 0),
            "hyena_mfma": (8 * M * D, 0), "rmsnorm": (4 * M * D, 0),
            "sum_norm": (12 * M * D, 0), "rglru_chunk_bf16": (6 * M * RGLRU["width"], 4 * M * RGLRU["width"] ** 2 // RGLRU["blocks"])}


def decode_work(B, ctx):
    l, H = LATENT, HEADS
    return {"lightning_recurrent": (8 * B * H * 128 * 128, 0), "latent_absorb": (2 * H * l["dim"] * l["kv_rank"], 0),
            "latent_decode": (2 * B * min(ctx, l["window"]) * (l["kv_rank"] + l["rot_dim"]), 0), "latent_up": (2 * H * l["vdim"] * l["kv_rank"], 0),
            "attn_decode": (B * ctx * H * 128 * 4, 0),
            "rglru_step_bf16": (RGLRU["width"] * (4 * RGLRU["width"] // RGLRU["blocks"] + B * 30), 0)}


def with_fractions(times, work):
    out = {}
    for k, (n, us) in sorted(times.items(), key=lambda kv: -kv[1][0] * kv[1][1]):
        out[k] = {"launches": n, "us": round(us, 2)}
        if k in work:
            b, f = work[k]
            out[k]["of_peak"] = round(max(b / HBM, f / MFMA) / (us * 1e-6), 3)
    return out


def captured(fn, n=20):
    """us per call inside a hipGraph (no event or host time between the launches)"""
    fn()
    torch.cuda.synchronize()
    g = torch.cuda.CUDAGraph()
    with torch.cuda.graph(g):
        for _ in range(n):
            fn()
    g.replay()
    torch.cuda.synchronize()
    best = 1e9
    for _ in range(3):
        a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
        a.record()
        g.replay()
        b.record()
        torch.cuda.synchronize()
        best = min(best, a.elapsed_time(b) / n * 1e3)
    return best


class Alone:
    """Kernels by themselves, without the rest of a model: {name: [us, fraction of peak]}."""

    def __init__(self, device):
        from evo_amd.ops import default_ops
        self.ops, self.device, self.out = default_ops(), device, {}

    def rnd(self, *shape):
        return torch.randn(*shape, device=self.device).to(torch.bfloat16)

    def put(self, name, fn, nbytes=0, flop=0, n=20):
        us = captured(fn, n)
        progress(f"{name}: {us:.1f} us")
        self.out[name] = [round(us, 1), round(max(nbytes / HBM, flop / MFMA) / (us * 1e-6), 3)]

    def pairs(self, B, T, heads, window=None, keep=0):
        """visible (query, key) pairs"""
        W = min(window or T, T)
        return B * heads * (W * (W + 1) // 2 + (T - W) * W + max(0, T - W) * min(keep, T - W) - min(keep, max(0, T - W)) * (min(keep, max(0, T - W)) - 1) // 2)

    def lightning(self, B, T, n=5):
        from evo_amd.mixer_ops import TokenBatch
        H = HEADS
        dec = torch.linspace(0.5, 0.999, H, device=self.device)
        batch = TokenBatch.of_prompts([T] * B, [0] * B, self.device)
        z, st = self.rnd(B * T, 4 * WIDTH), torch.zeros(B, H, 128, 128, device=self.device)
        self.put(f"lightning {B}x{T}", lambda: self.ops.lightning(z, H, 128, 128, dec, torch.log2(dec), batch, st), nbytes=8 * B * T * WIDTH, n=n)

    def latent_window(self, B, T, W):
        from evo_amd.mixer_ops import TokenBatch
        H, batch = HEADS, TokenBatch.of_prompts([T] * B, [0] * B, self.device)
        qd, kv, kr, sink = self.rnd(B * T, 6912), self.rnd(B * T, H * 256), self.rnd(B * T, 64), torch.zeros(H, device=self.device)
        self.put(f"window {B}x{T} w{W}", lambda: self.ops.window_attention(qd, kv, kr, H, 128, 64, 128, W, 0.07, sink, batch.cu, batch.cu, T),
                 flop=2 * 320 * self.pairs(B, T, H, W), n=3)

    def causal(self, B, T):
        qkv = self.rnd(B, T, 3, HEADS, 128)
        self.put(f"causal attention {B}x{T}", lambda: self.ops.attention(qkv[:, :, 0], qkv[:, :, 1], qkv[:, :, 2], 0), flop=2 * 256 * self.pairs(B, T, HEADS), n=3)

    def attention_decode(self, B, ctx):
        q, kv = self.rnd(B, 1, HEADS, 128), self.rnd(B, ctx, 2, HEADS, 128)
        self.put(f"attention decode {B}x{ctx}", lambda: self.ops.attention_decode(q, kv[:, :, 0], kv[:, :, 1]), nbytes=B * ctx * HEADS * 128 * 4)

    def lightning_step(self, B):
        from evo_amd.mixer_ops import TokenBatch
        H = HEADS
        dec = torch.linspace(0.5, 0.999, H, device=self.device)
        l2, batch = torch.log2(dec), TokenBatch.of_decode(torch.zeros(B, dtype=torch.int64, device=self.device))
        z, st = self.rnd(B, 4 * WIDTH), torch.zeros(B, H, 128, 128, device=self.device)
        self.put(f"lightning step {B}", lambda: self.ops.lightning(z, H, 128, 128, dec, l2, batch, st), nbytes=8 * B * H * 128 * 128)

    def latent_decode(self, B, ctx):
        from evo_amd.mixer_ops import MixerOps
        H, R = HEADS, LATENT["kv_rank"]
        cache, qd = self.rnd(B, ctx, MixerOps.latent_row(R, 64)), self.rnd(B, 6912)
        wuk, wuv, sink = self.rnd(H * 128, R), self.rnd(H * 128, R), torch.zeros(H, device=self.device)
        pos = torch.full((B,), 2 * ctx + 5, dtype=torch.int64, device=self.device)
        self.put(f"latent decode (three launches) {B}x{ctx}",
                 lambda: self.ops.latent_decode(qd, cache, pos, wuk, wuv, sink, H, 128, 64, 128, R, ctx, 0.07), nbytes=2 * B * ctx * 576 + 4 * H * 128 * R)

    def closing_norms(self, M):
        x, xb, y, w = torch.randn(M, WIDTH, device=self.device), self.rnd(M, WIDTH), self.rnd(M, WIDTH), self.rnd(WIDTH)
        self.put(f"norm then addition {M}", lambda: self.ops.postnorm_residual_(x, xb, y, w, 1e-6, 1.0), nbytes=12 * M * WIDTH)
        self.put(f"norm of the sum {M}", lambda: self.ops.sum_norm_(x, xb, y, w, 2.0, 1e-6, 0.0), nbytes=12 * M * WIDTH)

    def rglru_weights(self):
        W, nb = RGLRU["width"], RGLRU["blocks"]
        return (self.rnd(W, 4), self.rnd(W), self.rnd(nb, W // nb, W // nb) / 16, self.rnd(nb, W // nb), self.rnd(nb, W // nb, W // nb) / 16, self.rnd(nb, W // nb),
                -torch.rand(W, device=self.device))

    def rglru(self, B, T, n=5):
        from evo_amd.mixer_ops import TokenBatch
        W, nb = RGLRU["width"], RGLRU["blocks"]
        batch, w = TokenBatch.of_prompts([T] * B, [0] * B, self.device), self.rglru_weights()
        z, st = self.rnd(B * T, 2 * W), torch.zeros(B, 5, W, device=self.device)
        self.put(f"gated recurrence {B}x{T}", lambda: self.ops.rglru(z, None, False, W, *w, batch, st), nbytes=6 * B * T * W, flop=4 * B * T * W * (W // nb), n=n)

    def rglru_step(self, B):
        from evo_amd.mixer_ops import TokenBatch
        W, nb, w = RGLRU["width"], RGLRU["blocks"], self.rglru_weights()
        batch = TokenBatch.of_decode(torch.full((B,), 77, dtype=torch.int64, device=self.device))
        z, st, b = self.rnd(B, 2 * W), torch.zeros(B, 5, W, device=self.device), self.rnd(2 * W)
        self.put(f"gated recurrence step {B}", lambda: self.ops.rglru(z, b, True, W, *w, batch, st), nbytes=4 * W * (W // nb) + 30 * B * W)

    def heads(self, B, T, m, maps):
        from evo_amd.mixer_ops import TokenBatch
        H, G, n, dv, mask = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m.get("mask") or {}
        batch, nq, nk = TokenBatch.of_prompts([T] * B, [0] * B, self.device), H * maps, G * maps
        z, freq = self.rnd(B * T, (nq + nk) * n + G * dv), torch.rand(n // 2, device=self.device)
        what = f"{'two-map' if maps == 2 else 'grouped'} attention {B}x{T}" + (f" w{mask['size']}" if mask else "")
        W, keep = mask.get("size"), mask.get("keep_first", 0)
        self.put(what, lambda: self.ops.heads_attention(z, z[:, nq * n:], H, G, maps, n, dv, W, keep, n ** -0.5, 0.3, 0.5, 1e-6, batch.cu, batch.cu, T),
                 flop=2 * (n + dv) * maps * self.pairs(B, T, H, W, keep), n=3)
        cache = torch.zeros(B, keep + W if W else T, nk * n + G * dv, dtype=torch.bfloat16, device=self.device)
        rows = B * min(T, cache.shape[1])
        self.put(what.replace("attention", "preparation"), lambda: self.ops.heads_prep(z, nq, nk, n, G * dv, None, freq, 1.0, True, 1e-6, batch, cache, keep),
                 nbytes=B * T * (nq + nk) * n * 4 + rows * (nk * n * 2 + G * dv * 4))

    def heads_decode(self, B, ctx, m, maps):
        H, G, n, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        z, cache = self.rnd(B, (H + G) * maps * n + G * dv), self.rnd(B, ctx, G * (maps * n + dv))
        pos = torch.full((B,), 2 * ctx + 5, dtype=torch.int64, device=self.device)
        self.put(f"{'two-map' if maps == 2 else 'grouped'} attention decode (two launches) {B}x{ctx}",
                 lambda: self.ops.heads_decode(z, cache, pos, H, G, maps, n, dv, n ** -0.5, 0.3, 0.5, 1e-6), nbytes=2 * B * ctx * G * (maps * n + dv))


def kernels_alone(arch, device):
    """The attention, recurrence and decode kernels of a model and of the closest ones by themselves, at the same sequences."""
    a = Alone(device)
    with torch.inference_mode():
        for B, T in ((8, 2048), (1, 8192), (8, 8192)):
            a.lightning(B, T)
            for W in (1024, 4096):
                a.latent_window(B, T, W)
            a.causal(B, T)
            if arch == "batodra":
                a.rglru(B, T)
                for W in (1024, 4096):
                    a.heads(B, T, dict(WINDOWED, mask=dict(size=W, keep_first=4)), 1)
                a.heads(B, T, DIFFERENTIAL, 2)
            torch.cuda.empty_cache()
        for ctx in (1024, 4096):
            for B in (1, 8, 32):
                if arch == "vozalorn":
                    a.latent_decode(B, ctx)
                a.attention_decode(B, ctx)
                if arch == "batodra":
                    a.heads_decode(B, ctx, WINDOWED, 1)
                    a.heads_decode(B, ctx, DIFFERENTIAL, 2)
        for B in (1, 8, 32):
            a.lightning_step(B)
            if arch == "batodra":
                a.rglru_step(B)
        if arch == "batodra":
            a.closing_norms(16384)
    torch.cuda.empty_cache()
    return a.out


def run(device, arch="vozalorn", n_layers=8, steps=10):
    from evo_amd.pool import DecodePool
    from evo_amd.tokenizer import CharLevelTokenizer
    res = {"arch": arch, "width": WIDTH, "ff": FF, "layers": n_layers, "latent": LATENT, "lightning": LIGHT, "data": "synthetic", "dtype": "bf16"}
    if arch == "batodra":
        res.update(plain_ff=PLAIN_FF, windowed=WINDOWED, differential=DIFFERENTIAL, rglru=RGLRU)
    for kind in [arch] + BESIDE[arch]:
        m = build(kind, n_layers, device)
        r = res[kind] = {"weights_GB": round(weight_bytes(m) / 1e9, 3)}
        with torch.inference_mode():
            for B, T in ((8, 2048), (1, 8192), (8, 8192)):
                ids = torch.randint(0, 512, (B, T), device=device)
                s = seconds(lambda: m.hidden_states(ids), steps)
                r[f"prefill_{B}x{T}"] = {"tokens_per_s": round(B * T / s), "ms": round(s * 1e3, 3),
                                         "kernels": with_fractions(kernel_times(m, lambda: m.hidden_states(ids)), prefill_work(B, T))}
                progress(f"{kind} prefill {B} x {T}: {s * 1e3:.2f} ms")
            for B, ctx in ((1, 2048), (8, 2048), (32, 2048)):
                pool = DecodePool(m, CharLevelTokenizer(512), n_slots=B, device=device)
                first = pool.prefill([torch.randint(0, 512, (ctx,), device=device)])[0]
                slots = [pool.install(first, ctx, 256) for _ in range(B)]
                s = seconds(lambda: pool._advance(slots), 50, warmup=4)
                r[f"decode_{B}x{ctx}"] = {"tokens_per_s": round(B / s), "us_per_step": round(s * 1e6, 1),
                                          "weights_of_hbm_peak": round(weight_bytes(m) / s / HBM, 3), "captured": pool._graph is not None,
                                          "kernels": with_fractions(kernel_times(m, pool._step_eager), decode_work(B, ctx))}
                progress(f"{kind} decode {B} x {ctx}: {s * 1e6:.0f} us")
                del pool
        del m
        torch.cuda.empty_cache()
    res["kernels_alone_us_and_fraction_of_peak"] = kernels_alone(arch, device)
    return res


if __name__ == "__main__":
    print(json.dumps(run("cuda:0")))
