"""Small Batodra configurations and random weights for the tests, and the reference run on them (oracle/batodra_ref.py)."""
import json
import math

import torch

from oracle.batodra_ref import RefBatodra
from vozalorn_util import build, rel_err, rounding_noise, row_err, tokens  # noqa: F401


def recurrence(width=96, blocks=4, conv=4, ff=None):
    return dict(type="rglru", mixer=dict(width=width, blocks=blocks, conv=conv), mlp=None if ff is None else dict(kind="dense", ff=ff))


def differential(heads=2, kv_heads=2, dim=24, vdim=40, rot=8, base=9000.0, scale=None, diff=0.25, ff=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, rot=dict(base=base, dims=rot), scale=scale if scale is not None else 2.0 * dim ** -0.5, diff=diff)
    return dict(type="attention", mixer=m, mlp=None if ff is None else dict(kind="dense", ff=ff))


def windowed(heads=4, kv_heads=2, dim=32, vdim=24, rot=32, base=20000.0, window=9, keep=3, scale=None, factor=3.0, original=64, fast=8.0, slow=0.5, ff=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, mask=dict(size=window, keep_first=keep), scale=scale if scale is not None else 3.0 / dim ** 0.5,
             rot=dict(base=base, dims=rot, scaling=dict(factor=factor, original=original, fast=fast, slow=slow)))
    return dict(type="attention_2", mixer=m, mlp=None if ff is None else dict(kind="dense", ff=ff))


def again(layers, *which):
    """The layers, then some of them once more on the same tensors."""
    return layers + [dict(json.loads(json.dumps(layers[j])), weights_of=j) for j in which]


def config(layers, vocab=150, width=160, eps=1e-5, alpha=1.7):
    return dict(architecture="Batodra", vocab=vocab, width=width, norm=dict(eps=eps), postln_alpha=alpha, layers=layers)


# sizes, orders and constants of every kind: grouped heads, dims that are no multiple of 8 (or of anything), partial rotations, windows of one
# token up to several key tiles, kept tokens from none to more than the window, taps from one to five, feed-forwards missing, layers run again
CONFIGS = {
    "plain": config(again([windowed(ff=256), recurrence(ff=256), differential(ff=256)], 0, 1, 2)),
    "order": config(again([differential(heads=6, kv_heads=2, ff=96), recurrence(width=64, blocks=1), windowed(window=5, keep=0, ff=None),
                           windowed(heads=3, kv_heads=1, window=70, keep=66), recurrence(width=320, blocks=2, conv=2, ff=160)], 4, 0), alpha=0.8),
    "odd": config(again([windowed(heads=2, kv_heads=1, dim=10, vdim=9, rot=6, window=4, keep=1, ff=70), recurrence(width=54, blocks=3, conv=5, ff=51),
                         differential(heads=3, kv_heads=1, dim=7, vdim=11, rot=4, ff=33)], 2), vocab=101, width=100, eps=1e-3, alpha=2.6),
    "grouped": config([windowed(heads=36, kv_heads=2, dim=16, vdim=32, rot=16, window=40, keep=7, ff=384),
                       differential(heads=20, kv_heads=1, dim=8, vdim=16, rot=8, diff=0.6)], width=192, vocab=513, alpha=1.0),
    "window_1": config([windowed(window=1, keep=2), recurrence(width=128, blocks=1, conv=1, ff=128)], width=128, alpha=4.0),
    "window_64": config([windowed(window=64, keep=64, dim=64, vdim=64, rot=64, ff=128), recurrence(width=512, blocks=2, conv=3, ff=256),
                         differential(dim=64, vdim=128, rot=32)], width=256),
    "big_head": config([windowed(heads=2, kv_heads=2, dim=128, vdim=128, rot=64, window=100, keep=1), differential(heads=2, kv_heads=1, dim=128, vdim=256, rot=128),
                        recurrence(width=768, blocks=2)], width=128, alpha=1.2),
}


def shapes_of(cfg):
    """Tensor shapes restated from the configuration (not taken from the model class)."""
    D, V = cfg["width"], cfg["vocab"]
    out = {"embed": (V, D), "head": (V, D), "final.norm": (D,)}
    for i, l in enumerate(cfg["layers"]):
        if l.get("weights_of") is not None:
            continue
        m, p = l["mixer"], f"l{i}.mix."
        out[f"l{i}.norm1"] = (D,)
        if l["type"] == "rglru":
            W, nb = m["width"], m["blocks"]
            s = W // nb
            out.update({p + "y": (W, D), p + "y.b": (W,), p + "x": (W, D), p + "x.b": (W,), p + "conv": (W, m["conv"]), p + "conv.b": (W,), p + "ra": (nb, s, s),
                        p + "ra.b": (nb, s), p + "ri": (nb, s, s), p + "ri.b": (nb, s), p + "lam": (W,), p + "o": (D, W)})
        else:
            H, G, n, dv, k = m["heads"], m["kv_heads"], m["dim"], m["vdim"], 2 if l["type"] == "attention" else 1
            out.update({p + "q": (H * k * n, D), p + "k": (G * k * n, D), p + "v": (G * dv, D), p + "o": (D, H * dv)})
            if k == 2:
                out.update({p + t: (n,) for t in ("q.norm", "k.norm", "lq1", "lk1", "lq2", "lk2")})
        if l["mlp"]:
            F = l["mlp"]["ff"]
            out.update({f"l{i}.norm2": (D,), f"l{i}.mlp.up": (F, D), f"l{i}.mlp.down": (D, F)})
    return out


def weights(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, s in shapes_of(cfg).items():
        t = torch.randn(*s, generator=g)
        if "norm" in name:
            t = 1.0 + 0.3 * t
        elif name.endswith("lam"):
            t = t * 1.5 - 3.0                                     # decays from 1 - 1e-3 to a half
        elif name[-3:] in ("lq1", "lk1", "lq2", "lk2"):
            t = t * 0.2
        elif name.endswith("conv"):
            t = t * 0.6
        elif name.endswith(".b"):
            t = t * 0.5
        elif name != "embed":
            t = t * (1.4 / math.sqrt(s[-1]))
        out[name] = t.to(torch.bfloat16)
    return out


def reference(cfg, w):
    return RefBatodra(cfg, w, torch.float64)


def spiky(cfg, w, token=7, gain=6.0):
    """The weights with one token whose key stands out for every query of the attention layers: where it is seen, it takes most of the
    weight, so a window's, a kept token's or a page's edge off by one moves the logits by their full size.  A shared direction e of the
    stream is in every embedding (queries) and, larger, in this token's (key)."""
    w = {k: t.clone() for k, t in w.items()}
    D = cfg["width"]
    e = torch.zeros(D)
    e[0] = 1.0
    w["embed"][:, 0] = 3.0
    w["embed"][token, 0] = 3.0 * gain
    for i, l in enumerate(cfg["layers"][:1]):
        m = l["mixer"]
        n, k = m["dim"], 2 if l["type"] == "attention" else 1
        last = n - 1                                              # the slowest pair's second half, or a dimension that is not rotated
        for name, heads in (("q", m["heads"] * k), ("k", m["kv_heads"] * k)):
            t = w[f"l{i}.mix.{name}"].view(heads, n, D)
            t[:, last, 0] += 3.0
    return w
