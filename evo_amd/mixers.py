"""Sublayers of the models that a config.json describes layer by layer: token mixers and feed-forwards.

A sublayer names its checkpoint tensors (`tensors`), keeps them fused the way the launches read them -- the state dict comes back as views
of the fused storage, one weight set --, and runs on packed tokens (evo_amd/mixer_ops.py TokenBatch).  A mixer says where its per-sequence
state lives in the inference-parameter records (`store`), how one row of it looks (`new_cache`) and whether it grows with the sequence
(`grows`).  Sizes and constants are parameters; a model class lists the kinds it has (evo_amd/decoder.py).
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch
import torch.nn as nn

from .mixer_ops import Stream, TokenBatch


def _need(cfg: dict, key: str, where: str):
    if key not in cfg:
        raise ValueError(f"{where}: '{key}' is missing")
    return cfg[key]


def _size(cfg: dict, key: str, where: str) -> int:
    v = _need(cfg, key, where)
    if int(v) != v or int(v) <= 0:
        raise ValueError(f"{where}: '{key}' must be a positive integer, got {v!r}")
    return int(v)


class Sublayer(nn.Module):
    """`tensors`: {name: shape} of the checkpoint; `_fuse(named)` sets the buffers; `_views()` gives the checkpoint tensors back."""

    def __init__(self, dtype: torch.dtype):
        super().__init__()
        self.dtype = dtype

    def tensors(self) -> Dict[str, tuple]:
        raise NotImplementedError

    grows = False                # a mixer's cache holds every token ([rows, positions, ..]) rather than a fixed state

    def load(self, named: Dict[str, torch.Tensor]) -> None:
        for k, t in self._fuse({k: t.detach() for k, t in named.items()}).items():
            self.register_buffer(k, t.contiguous(), persistent=False)

    def _stack(self, *parts: torch.Tensor) -> torch.Tensor:
        """Weights that share their input, one below the other: one matrix product.  Wide stacks are padded with zero rows to whole
        256-row tiles (csrc/gemm.hip); what reads the product ignores the extra columns."""
        w = torch.cat([p.to(self.dtype) for p in parts])
        pad = -w.shape[0] % 256
        if self.dtype == torch.bfloat16 and w.shape[0] >= 1024 and w.shape[1] % 64 == 0 and pad:
            w = torch.cat([w, w.new_zeros(pad, w.shape[1])])
        return w


class LightningMixer(Sublayer):
    """Linear attention with one constant decay per head; the concatenated heads are RMS-normed together and gated before the output
    projection.  Per-sequence state: [heads, dim, vdim] fp32 in the recurrent record."""

    def __init__(self, cfg: dict, width: int, eps: float, dtype: torch.dtype, where: str):
        super().__init__(dtype)
        self.heads, self.dk, self.dv = (_size(cfg, k, where) for k in ("heads", "dim", "vdim"))
        decay = [float(a) for a in _need(cfg, "decay", where)]
        if len(decay) != self.heads or not all(0.0 <= a <= 1.0 for a in decay):
            raise ValueError(f"{where}: 'decay' must hold one value in [0, 1] per head")
        self.width, self.eps = width, eps
        self.register_buffer("decay", torch.tensor(decay, dtype=torch.float32), persistent=False)
        self.register_buffer("log2_decay", torch.tensor([math.log2(a) if a > 0 else -math.inf for a in decay], dtype=torch.float32), persistent=False)

    def tensors(self):
        D, H, dk, dv = self.width, self.heads, self.dk, self.dv
        return {"q": (H * dk, D), "k": (H * dk, D), "v": (H * dv, D), "g": (H * dv, D), "o": (D, H * dv), "norm": (H * dv,)}

    def _fuse(self, t):
        return {"w_in": self._stack(t["q"], t["k"], t["v"], t["g"]), "w_o": t["o"].to(self.dtype), "w_norm": t["norm"].to(self.dtype)}

    def _views(self):
        nk, nv = self.heads * self.dk, self.heads * self.dv
        q, k, v, g = self.w_in[: 2 * nk + 2 * nv].split([nk, nk, nv, nv])
        return {"q": q, "k": k, "v": v, "g": g, "o": self.w_o, "norm": self.w_norm}

    def dense_shapes(self):
        return [tuple(self.w_in.shape), tuple(self.w_o.shape)]

    @staticmethod
    def store(ipd: dict) -> dict:
        return ipd["hyena"].state_dict

    def new_cache(self, rows: int, device, capacity: int = 0) -> torch.Tensor:
        return torch.zeros(rows, self.heads, self.dk, self.dv, dtype=torch.float32, device=device)

    def mix(self, ops, stream: Stream, batch: TokenBatch, cache: Optional[torch.Tensor]) -> torch.Tensor:
        H, dk, dv = self.heads, self.dk, self.dv
        g0 = H * (2 * dk + dv)
        # [q | k | v | g]; a prompt's q, k, v come activated, a decode step activates its own
        z = stream.linear(self.w_in) if batch.decode else ops.linear_act(stream.input(), self.w_in, "silu", g0)
        o = ops.lightning(z, H, dk, dv, self.decay, self.log2_decay, batch, cache)
        return ops.linear(ops.gated_norm(o, z[:, g0:g0 + H * dv], self.w_norm, self.eps), self.w_o)


class LatentAttention(Sublayer):
    """Attention whose keys and values are linear maps of one cached latent per token, with a rotated key part shared by the heads, a
    sliding window and a sink per head.  Per-sequence state: a ring of `window` rows [latent | rotated key | zeros] in the KV record."""

    def __init__(self, cfg: dict, width: int, eps: float, dtype: torch.dtype, where: str):
        super().__init__(dtype)
        self.heads, self.dn, self.dr, self.dv, self.R = (_size(cfg, k, where) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
        self.scale = float(_need(cfg, "scale", where))
        self.window = _size(_need(cfg, "mask", where), "size", where + ".mask")
        rot = _need(cfg, "rot", where)
        self.n_rot = _size(rot, "dims", where + ".rot")
        if self.n_rot % 2 or self.n_rot > self.dr:
            raise ValueError(f"{where}.rot: 'dims' must be even and at most rot_dim")
        base = float(_need(rot, "base", where + ".rot"))
        self.width, self.eps = width, eps
        self.register_buffer("inv_freq", torch.tensor([base ** (-2.0 * i / self.n_rot) for i in range(self.n_rot // 2)], dtype=torch.float64)
                             .to(torch.float32), persistent=False)

    def tensors(self):
        D, H = self.width, self.heads
        return {"q": (H * (self.dn + self.dr), D), "dkv": (self.R + self.dr, D), "dkv.norm": (self.R,), "uk": (H * self.dn, self.R),
                "uv": (H * self.dv, self.R), "sink": (H,), "o": (D, H * self.dv)}

    def _fuse(self, t):
        return {"w_in": self._stack(t["q"], t["dkv"]), "w_norm": t["dkv.norm"].to(self.dtype),
                "w_kv": torch.cat([t["uk"], t["uv"]]).to(self.dtype), "sink": t["sink"].to(torch.float32), "w_o": t["o"].to(self.dtype)}

    def _views(self):
        nq, n = self.heads * (self.dn + self.dr), self.R + self.dr
        uk, uv = self.w_kv.split([self.heads * self.dn, self.heads * self.dv])
        return {"q": self.w_in[:nq], "dkv": self.w_in[nq:nq + n], "dkv.norm": self.w_norm, "uk": uk, "uv": uv, "sink": self.sink, "o": self.w_o}

    def dense_shapes(self):
        return [tuple(self.w_in.shape), tuple(self.w_o.shape)]

    @staticmethod
    def store(ipd: dict) -> dict:
        return ipd["mha"].key_value_memory_dict

    def new_cache(self, rows: int, device, capacity: int = 0) -> torch.Tensor:
        from .mixer_ops import MixerOps
        return torch.zeros(rows, self.window, MixerOps.latent_row(self.R, self.dr), dtype=self.dtype, device=device)

    def _earlier(self, batch: TokenBatch, cache: torch.Tensor):
        """Cached rows the first new token of every sequence still sees, oldest first -> ([rows, row], count per sequence)."""
        seen = [min(p, self.window - 1) for p in batch.past]
        b = torch.tensor([i for i, n in enumerate(seen) for _ in range(n)], dtype=torch.int64, device=cache.device)
        slot = torch.tensor([j % cache.shape[1] for p, n in zip(batch.past, seen) for j in range(p - n, p)], dtype=torch.int64, device=cache.device)
        return cache[b, slot], seen

    def mix(self, ops, stream: Stream, batch: TokenBatch, cache: Optional[torch.Tensor]) -> torch.Tensor:
        H, dn, dr, dv, R = self.heads, self.dn, self.dr, self.dv, self.R
        qd = stream.linear(self.w_in)                             # [queries | latent, shared key]
        if batch.decode:
            ops.latent_prep(qd, H, dn, dr, R, self.w_norm, self.inv_freq, self.eps, batch, cache, want_kv=False)
            a = ops.latent_decode(qd, cache, batch.pos, self.w_kv[:H * dn], self.w_kv[H * dn:], self.sink, H, dn, dr, dv, R, self.window, self.scale)
            return ops.linear(a, self.w_o)
        old, seen = (None, None) if batch.resume is None else self._earlier(batch, cache)   # (read before the ring moves on)
        c, kr = ops.latent_prep(qd, H, dn, dr, R, self.w_norm, self.inv_freq, self.eps, batch, cache, want_kv=True)
        cu_k = batch.cu
        if old is not None:
            olds, cs, krs = old.split(seen), c.split(batch.lens), kr.split(batch.lens)
            c = torch.cat([t for o, n in zip(olds, cs) for t in (o[:, :R], n)])
            kr = torch.cat([t for o, n in zip(olds, krs) for t in (o[:, R:R + dr], n)])
            total = torch.tensor([0] + [s + n for s, n in zip(seen, batch.lens)]).cumsum(0)
            cu_k = total.to(torch.int32).to(c.device)
        kv = ops.linear(c, self.w_kv)                             # every head's keys, then every head's values
        a = ops.window_attention(qd, kv, kr, H, dn, dr, dv, self.window, self.scale, self.sink, batch.cu, cu_k, max(batch.lens))
        return ops.linear(a, self.w_o)


def rotation(rot: dict, where: str):
    """A config's rotary part -> (frequency of every pair, factor on cosine and sine).  With `scaling` (factor, original, fast, slow) the pairs
    that turn fewer than `slow` times over the `original` length are slowed by `factor`, those with more than `fast` turns stay, the others
    lie on a ramp over the pair index (YaRN)."""
    n, base = _size(rot, "dims", where), float(_need(rot, "base", where))
    if n % 2:
        raise ValueError(f"{where}: 'dims' must be even")
    freq, amp = [base ** (-2.0 * i / n) for i in range(n // 2)], 1.0
    s = rot.get("scaling")
    if s is not None:
        factor, original, fast, slow = (float(_need(s, k, where + ".scaling")) for k in ("factor", "original", "fast", "slow"))

        def pair(turns):                                          # (not an integer) index of the pair that turns so often over the original length
            return n * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
        lo, hi = max(math.floor(pair(fast)), 0), min(math.ceil(pair(slow)), n - 1)
        ramp = [min(max((i - lo) / max(hi - lo, 1e-3), 0.0), 1.0) for i in range(n // 2)]
        freq = [f / factor * r + f * (1.0 - r) for f, r in zip(freq, ramp)]
        amp = 0.1 * math.log(factor) + 1.0
    return torch.tensor(freq, dtype=torch.float64).to(torch.float32), amp


class HeadAttention(Sublayer):
    """Softmax attention with one cached key and value per token and key head; query heads share key heads in groups.  Options:
      maps = 2   differential attention: two attention maps over the same values, their weighted difference normed per head
      qk_norm    RMS norms with a weight on queries and keys, before the rotation
      unit_qk    queries and keys divided by their root mean square, behind the rotation
      mask       a sliding window (`size`) whose first `keep_first` tokens stay visible; without it every earlier token is seen
    Per-sequence state in the KV record: rows [keys | values] per token, all of them or a ring of keep_first + size."""

    def __init__(self, cfg: dict, width: int, eps: float, dtype: torch.dtype, where: str, maps: int = 1, qk_norm: bool = False, unit_qk: bool = False):
        super().__init__(dtype)
        self.heads, self.kv_heads, self.dim, self.dv = (_size(cfg, k, where) for k in ("heads", "kv_heads", "dim", "vdim"))
        if self.heads % self.kv_heads:
            raise ValueError(f"{where}: 'heads' must be a multiple of 'kv_heads'")
        self.maps, self.qk_norm, self.unit_qk = maps, qk_norm, unit_qk
        self.scale = float(_need(cfg, "scale", where))
        self.diff = float(_need(cfg, "diff", where)) if maps == 2 else 0.0
        self.lam = 0.0                                            # weight of the second map: a function of the loaded vectors
        freq, self.amp = rotation(_need(cfg, "rot", where), where + ".rot")
        if 2 * freq.numel() > self.dim:
            raise ValueError(f"{where}.rot: 'dims' must be at most 'dim'")
        self.register_buffer("inv_freq", freq, persistent=False)
        mask = cfg.get("mask")
        self.window, self.keep = None, 0
        if mask is not None:
            self.window, self.keep = _size(mask, "size", where + ".mask"), int(mask.get("keep_first") or 0)
            if self.keep < 0:
                raise ValueError(f"{where}.mask: 'keep_first' must not be negative")
        self.grows = self.window is None
        self.width, self.eps = width, eps
        self.nq, self.nk, self.nv = self.heads * maps, self.kv_heads * maps, self.kv_heads * self.dv    # query and key vectors, values

    def tensors(self):
        D, n = self.width, self.dim
        out = {"q": (self.nq * n, D), "k": (self.nk * n, D), "v": (self.nv, D), "o": (D, self.heads * self.dv)}
        if self.qk_norm:
            out.update({"q.norm": (n,), "k.norm": (n,)})
        if self.maps == 2:
            out.update({k: (n,) for k in ("lq1", "lk1", "lq2", "lk2")})
        return out

    def _fuse(self, t):
        out = {"w_in": self._stack(t["q"], t["k"], t["v"]), "w_o": t["o"].to(self.dtype)}
        if self.qk_norm:
            out.update({"q_norm": t["q.norm"].to(self.dtype), "k_norm": t["k.norm"].to(self.dtype)})
        if self.maps == 2:
            out["l_vec"] = torch.stack([t[k] for k in ("lq1", "lk1", "lq2", "lk2")]).to(self.dtype)
            a, b, c, d = out["l_vec"].double().cpu()
            self.lam = float(torch.exp((a * b).sum()) - torch.exp((c * d).sum())) + self.diff
        return out

    def _views(self):
        q, k, v = self.w_in[: (self.nq + self.nk) * self.dim + self.nv].split([self.nq * self.dim, self.nk * self.dim, self.nv])
        out = {"q": q, "k": k, "v": v, "o": self.w_o}
        if self.qk_norm:
            out.update({"q.norm": self.q_norm, "k.norm": self.k_norm})
        if self.maps == 2:
            out.update(zip(("lq1", "lk1", "lq2", "lk2"), self.l_vec))
        return out

    def dense_shapes(self):
        return [tuple(self.w_in.shape), tuple(self.w_o.shape)]

    @staticmethod
    def store(ipd: dict) -> dict:
        return ipd["mha"].key_value_memory_dict

    def new_cache(self, rows: int, device, capacity: int = 0) -> torch.Tensor:
        row = (self.nk * self.dim + self.nv + 7) // 8 * 8         # (whole 16-byte pieces)
        return torch.zeros(rows, max(1, capacity) if self.grows else self.keep + self.window, row, dtype=self.dtype, device=device)

    def _earlier(self, batch: TokenBatch, cache: torch.Tensor):
        """Cached rows the first new token of every sequence still sees, oldest first -> one [rows, row] per sequence."""
        out = []
        for b, p in enumerate(batch.past):
            if self.window is None:
                out.append(cache[b, :p])
                continue
            kept, first = min(self.keep, p), max(self.keep, p - self.window + 1)
            slots = torch.cat([torch.arange(kept), self.keep + (torch.arange(first, max(first, p)) - self.keep) % self.window])
            out.append(cache[b, slots.to(cache.device)])
        return out

    def mix(self, ops, stream: Stream, batch: TokenBatch, cache: Optional[torch.Tensor]) -> torch.Tensor:
        H, G, n, dv = self.heads, self.kv_heads, self.dim, self.dv
        z = stream.linear(self.w_in)                              # [queries | keys | values]
        old = None if batch.decode or batch.resume is None else self._earlier(batch, cache)     # (read before the ring moves on)
        ops.heads_prep(z, self.nq, self.nk, n, self.nv, (self.q_norm, self.k_norm) if self.qk_norm else None, self.inv_freq, self.amp, self.unit_qk, self.eps,
                       batch, cache, self.keep)
        tail = (self.scale, self.lam, 1.0 - self.diff, self.eps)
        if batch.decode:
            return ops.linear(ops.heads_decode(z, cache, batch.pos, H, G, self.maps, n, dv, *tail), self.w_o)
        kv, cu_k = z[:, self.nq * n: (self.nq + self.nk) * n + self.nv], batch.cu
        if old is not None:
            kv = torch.cat([t for o, new in zip(old, kv.split(batch.lens)) for t in (o[:, : kv.shape[1]], new)])
            cu_k = torch.tensor([0] + [o.shape[0] + m for o, m in zip(old, batch.lens)]).cumsum(0).to(torch.int32).to(z.device)
        a = ops.heads_attention(z, kv, H, G, self.maps, n, dv, self.window, self.keep, *tail, batch.cu, cu_k, max(batch.lens))
        return ops.linear(a, self.w_o)


class GatedRecurrence(Sublayer):
    """A real-gated linear recurrence behind a short causal convolution, its output gated by a second branch (Griffin's recurrent block):
    a = exp(-c r softplus(lam)), S <- a S + sqrt(1 - a^2) i u, with the gates r and i from block-diagonal maps of u.  Per-sequence state in the
    recurrent record: [1 + taps, width] fp32 -- S, then a ring of the convolution's last inputs."""

    def __init__(self, cfg: dict, width: int, eps: float, dtype: torch.dtype, where: str, c: float = 8.0):
        super().__init__(dtype)
        self.W, self.blocks, self.taps = (_size(cfg, k, where) for k in ("width", "blocks", "conv"))
        if self.W % self.blocks:
            raise ValueError(f"{where}: 'width' must be a multiple of 'blocks'")
        self.width, self.c = width, c

    def tensors(self):
        D, W, nb, bs = self.width, self.W, self.blocks, self.W // self.blocks
        return {"y": (W, D), "y.b": (W,), "x": (W, D), "x.b": (W,), "conv": (W, self.taps), "conv.b": (W,), "ra": (nb, bs, bs), "ra.b": (nb, bs),
                "ri": (nb, bs, bs), "ri.b": (nb, bs), "lam": (W,), "o": (D, W)}

    def _fuse(self, t):
        out = {"w_in": self._stack(t["y"], t["x"]), "w_o": t["o"].to(self.dtype), "lam": t["lam"].to(self.dtype)}
        b = torch.cat([t["y.b"], t["x.b"]]).to(self.dtype)
        out["b_in"] = torch.cat([b, b.new_zeros(out["w_in"].shape[0] - b.numel())])
        out.update({k: t[n].to(self.dtype) for k, n in (("conv", "conv"), ("conv_b", "conv.b"), ("ra", "ra"), ("ra_b", "ra.b"), ("ri", "ri"), ("ri_b", "ri.b"))})
        out["decay"] = (-self.c * torch.nn.functional.softplus(out["lam"].double())).to(torch.float32)
        return out

    def _views(self):
        W = self.W
        return {"y": self.w_in[:W], "y.b": self.b_in[:W], "x": self.w_in[W:2 * W], "x.b": self.b_in[W:2 * W], "conv": self.conv, "conv.b": self.conv_b,
                "ra": self.ra, "ra.b": self.ra_b, "ri": self.ri, "ri.b": self.ri_b, "lam": self.lam, "o": self.w_o}

    def dense_shapes(self):
        return [tuple(self.w_in.shape), tuple(self.w_o.shape)]

    @staticmethod
    def store(ipd: dict) -> dict:
        return ipd["hyena"].state_dict

    def new_cache(self, rows: int, device, capacity: int = 0) -> torch.Tensor:
        return torch.zeros(rows, 1 + self.taps, self.W, dtype=torch.float32, device=device)

    def mix(self, ops, stream: Stream, batch: TokenBatch, cache: Optional[torch.Tensor]) -> torch.Tensor:
        # [y | x]; a prompt's come with their bias and activation, a decode step adds its own
        z = stream.linear(self.w_in) if batch.decode else ops.linear_act(stream.input(), self.w_in, "gelu_tanh", self.W, self.b_in)
        o = ops.rglru(z, self.b_in if batch.decode else None, batch.decode, self.W, self.conv, self.conv_b, self.ra, self.ra_b, self.ri, self.ri_b, self.decay,
                      batch, cache)
        return ops.linear(o, self.w_o)


class PlainFF(Sublayer):
    """W_down act(W_up x); a wide inner size is padded with zeros to whole 256-column tiles (csrc/gemm.hip)."""

    def __init__(self, cfg: dict, width: int, dtype: torch.dtype, where: str, act: str = "relu2"):
        super().__init__(dtype)
        self.width, self.ff, self.act = width, _size(cfg, "ff", where), act

    def tensors(self):
        return {"up": (self.ff, self.width), "down": (self.width, self.ff)}

    def _fuse(self, t):
        up, down = self._stack(t["up"]), t["down"].to(self.dtype)
        return {"w_up": up, "w_down": torch.cat([down, down.new_zeros(self.width, up.shape[0] - self.ff)], 1)}

    def _views(self):
        return {"up": self.w_up[:self.ff], "down": self.w_down[:, :self.ff]}

    def dense_shapes(self):
        return [tuple(self.w_up.shape), tuple(self.w_down.shape)]

    def forward_ff(self, ops, stream: Stream) -> torch.Tensor:
        return ops.linear(stream.linear(self.w_up, act=self.act), self.w_down)


class GatedFF(Sublayer):
    """W_down(silu(W_gate x) * (W_up x)); gate and up rows are kept in the gated launch's interleaved order where its shape allows."""

    def __init__(self, cfg: dict, width: int, dtype: torch.dtype, where: str):
        super().__init__(dtype)
        self.width, self.ff = width, _size(cfg, "ff", where)
        self.grouped = dtype == torch.bfloat16 and self.ff % 128 == 0 and width % 64 == 0 and width >= 128

    def tensors(self):
        return {"gate": (self.ff, self.width), "up": (self.ff, self.width), "down": (self.width, self.ff)}

    def _fuse(self, t):
        from .ops import HipOps
        w = torch.cat([t["gate"], t["up"]]).to(self.dtype)
        return {"w12": HipOps.pack_gate_weights(w) if self.grouped else w, "w3": t["down"].to(self.dtype)}

    def _views(self):
        w = self.w12
        if self.grouped:
            w = w.view(-1, 2, 32, self.width).transpose(0, 1).reshape(2 * self.ff, self.width)
        return {"gate": w[:self.ff], "up": w[self.ff:], "down": self.w3}

    def dense_shapes(self):
        return [tuple(self.w12.shape), tuple(self.w3.shape)]

    def forward_ff(self, ops, stream: Stream) -> torch.Tensor:
        return ops.linear(stream.gate(self.w12, self.grouped, "silu"), self.w3)


def build_mixer(kinds: dict, layer: dict, width: int, eps: float, dtype: torch.dtype, where: str) -> Sublayer:
    kind = _need(layer, "type", where)
    if kind not in kinds:
        raise ValueError(f"{where}: unknown mixer '{kind}' (known: {', '.join(kinds)})")
    return kinds[kind](_need(layer, "mixer", where), width, eps, dtype, f"{where}.mixer")


def build_feed_forward(kinds: dict, layer: dict, width: int, dtype: torch.dtype, where: str) -> Optional[Sublayer]:
    mlp = layer.get("mlp")
    if mlp is None:
        return None
    kind = _need(mlp, "kind", f"{where}.mlp")
    if kind not in kinds:
        raise ValueError(f"{where}: unknown feed-forward '{kind}' (known: {', '.join(kinds)})")
    return kinds[kind](mlp, width, dtype, f"{where}.mlp")
