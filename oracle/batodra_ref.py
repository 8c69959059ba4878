"""Plain restatement of the Batodra decoder, one function per mechanism, token by token where the mechanism is a recurrence.

TEST INFRASTRUCTURE: shares no code with evo_amd.  Everything runs in the dtype of the tensors it is given (the tests use float64);
a sequence is a [T, width] matrix, a model is (config dict, {tensor name: tensor}).
"""
import math
from typing import Dict, Optional

import torch


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x, w, eps):
    return unit_rms(x, eps) * w


def norm_of_sum(x, y, alpha, w, eps):
    """The layer's norm sits behind the addition: N(alpha x + y)."""
    return rms_norm(alpha * x + y, w, eps)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def squared_relu(z):
    return torch.clamp(z, min=0.0) ** 2


def rotation_frequencies(base: float, dims: int):
    return [base ** (-2.0 * i / dims) for i in range(dims // 2)]


def yarn(freqs, base: float, dims: int, factor: float, original: float, fast: float, slow: float):
    """-> (frequencies, amplitude): pairs that turn fewer than `slow` times over `original` positions are slowed by `factor`, those above
    `fast` turns stay, a linear ramp over the pair index lies between."""
    def pair_of(turns):
        return dims * math.log(original / (2 * math.pi * turns)) / (2 * math.log(base))
    lo, hi = max(math.floor(pair_of(fast)), 0), min(math.ceil(pair_of(slow)), dims - 1)
    out = []
    for i, f in enumerate(freqs):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / factor * r + f * (1 - r))
    return out, 0.1 * math.log(factor) + 1.0


def rotate(x, pos, freqs, amplitude: float = 1.0):
    """x [T, heads, n]: elements (i, i + len(freqs)) turned by pos * freqs[i] and scaled by the amplitude; the rest unchanged."""
    half = len(freqs)
    a = pos.to(x.dtype)[:, None, None] * torch.tensor(freqs, dtype=x.dtype)
    c, s = a.cos() * amplitude, a.sin() * amplitude
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * half:]], -1)


def visible(q_pos, k_pos, window: Optional[int] = None, keep_first: int = 0):
    d = q_pos[:, None] - k_pos[None, :]
    ok = d >= 0
    if window is not None:
        ok = ok & ((d < window) | (k_pos[None, :] < keep_first))
    return ok


def softmax_attention(q, k, v, scale: float, mask):
    """q [Tq, H, n], k [Tk, G, n], v [Tk, G, dv] -> [Tq, H, dv]; query head h reads key head h // (H / G)."""
    H, G = q.shape[1], k.shape[1]
    out = []
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale
        p = torch.softmax(s.masked_fill(~mask, -math.inf), -1)
        out.append(p @ v[:, g])
    return torch.stack(out, 1)


def difference_of_maps(a1, a2, lam, diff: float, eps: float):
    return unit_rms(a1 - lam * a2, eps) * (1.0 - diff)


def difference_weight(w, diff: float):
    return torch.exp((w["lq1"] * w["lk1"]).sum()) - torch.exp((w["lq2"] * w["lk2"]).sum()) + diff


def differential_attention_mixer(h, m: dict, w: Dict[str, torch.Tensor], eps: float, past=None):
    """`past`: (keys of both maps [P, G, 2, n], values [P, G, dv]) of earlier tokens.  Returns (output, the same of all tokens)."""
    T, H, G, n, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    P = 0 if past is None else past[0].shape[0]
    pos = torch.arange(P, P + T)
    f = rotation_frequencies(m["rot"]["base"], m["rot"]["dims"])
    q = rms_norm((h @ w["q"].T).view(T, H * 2, n), w["q.norm"], eps)
    k = rms_norm((h @ w["k"].T).view(T, G * 2, n), w["k.norm"], eps)
    q, k = rotate(q, pos, f).view(T, H, 2, n), rotate(k, pos, f).view(T, G, 2, n)
    v = (h @ w["v"].T).view(T, G, dv)
    if past is not None:
        k, v = torch.cat([past[0], k]), torch.cat([past[1], v])
    mask = visible(pos, torch.arange(P + T))
    a1, a2 = (softmax_attention(q[:, :, i], k[:, :, i], v, m["scale"], mask) for i in (0, 1))
    o = difference_of_maps(a1, a2, difference_weight(w, m["diff"]), m["diff"], eps)
    return o.reshape(T, H * dv) @ w["o"].T, (k, v)


def windowed_attention_mixer(h, m: dict, w: Dict[str, torch.Tensor], eps: float, past=None):
    T, H, G, n, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    P = 0 if past is None else past[0].shape[0]
    pos = torch.arange(P, P + T)
    r = m["rot"]
    f, amp = yarn(rotation_frequencies(r["base"], r["dims"]), r["base"], r["dims"], **r["scaling"])
    q = unit_rms(rotate((h @ w["q"].T).view(T, H, n), pos, f, amp), eps)
    k = unit_rms(rotate((h @ w["k"].T).view(T, G, n), pos, f, amp), eps)
    v = (h @ w["v"].T).view(T, G, dv)
    if past is not None:
        k, v = torch.cat([past[0], k]), torch.cat([past[1], v])
    o = softmax_attention(q, k, v, m["scale"], visible(pos, torch.arange(P + T), m["mask"]["size"], m["mask"]["keep_first"]))
    return o.reshape(T, H * dv) @ w["o"].T, (k, v)


def causal_convolution(x, taps, bias, before=None):
    """x [T, C], taps [C, n] (last column: the current token) -> (u [T, C], the last n - 1 inputs)."""
    T, n = x.shape[0], taps.shape[1]
    before = torch.zeros(n - 1, x.shape[1], dtype=x.dtype) if before is None else before
    z = torch.cat([before, x])
    u = sum(z[i:i + T] * taps[:, i] for i in range(n)) + bias
    return u, z[T:]


def block_diagonal(u, m, b):
    """u [T, W] in B parts, m [B, s, s], b [B, s]."""
    B, s, _ = m.shape
    return torch.cat([u[:, i * s:(i + 1) * s] @ m[i].T + b[i] for i in range(B)], -1)


def gated_linear_recurrence(u, r, i, lam, state=None):
    """-> (S of every token [T, W], last S):  log a = -8 r softplus(lam),  S <- a S + sqrt(1 - a^2) i u."""
    log_a = -8.0 * r * torch.log1p(torch.exp(lam))
    a = torch.exp(log_a)
    add = torch.sqrt(-torch.expm1(2.0 * log_a)) * i * u
    S = torch.zeros_like(u[0]) if state is None else state
    out = []
    for t in range(u.shape[0]):
        S = a[t] * S + add[t]
        out.append(S)
    return torch.stack(out), S


def recurrent_mixer(h, m: dict, w: Dict[str, torch.Tensor], eps: float, past=None):
    """`past`: (last convolution inputs, S)."""
    y = gelu_tanh(h @ w["y"].T + w["y.b"])
    u, tail = causal_convolution(h @ w["x"].T + w["x.b"], w["conv"], w["conv.b"], None if past is None else past[0])
    r = torch.sigmoid(block_diagonal(u, w["ra"], w["ra.b"]))
    i = torch.sigmoid(block_diagonal(u, w["ri"], w["ri.b"]))
    S, last = gated_linear_recurrence(u, r, i, w["lam"], None if past is None else past[1])
    return (S * y) @ w["o"].T, (tail, last)


def feed_forward(h, w):
    return squared_relu(h @ w["up"].T) @ w["down"].T


MIXERS = {"rglru": recurrent_mixer, "attention": differential_attention_mixer, "attention_2": windowed_attention_mixer}


class RefBatodra:
    """`ref(ids)` -> logits [T, vocab] of one sequence.  `carry` (a dict) keeps the mixers' state between calls."""

    def __init__(self, config: dict, tensors: Dict[str, torch.Tensor], dtype=torch.float64):
        self.config = config
        self.w = {k: t.to(dtype) for k, t in tensors.items()}

    def _sub(self, prefix):
        return {k[len(prefix):]: t for k, t in self.w.items() if k.startswith(prefix)}

    def __call__(self, ids, carry: Optional[dict] = None, taps: Optional[list] = None):
        c = self.config
        eps, alpha = c["norm"]["eps"], c["postln_alpha"]
        x = self.w["embed"][torch.as_tensor(ids)]
        for i, layer in enumerate(c["layers"]):
            j = layer.get("weights_of", i)
            state = None if carry is None else carry.get(i)
            y, state = MIXERS[layer["type"]](x, layer["mixer"], self._sub(f"l{j}.mix."), eps, state)
            if carry is not None:
                carry[i] = state
            x = norm_of_sum(x, y, alpha, self.w[f"l{j}.norm1"], eps)
            if layer.get("mlp") is not None:
                x = norm_of_sum(x, feed_forward(x, self._sub(f"l{j}.mlp.")), alpha, self.w[f"l{j}.norm2"], eps)
            if taps is not None:
                taps.append(x)
        return rms_norm(x, self.w["final.norm"], eps) @ self.w["head"].T
