"""The mixer libraries (include/evo_mi355x.h, last section) as methods of the op set: kernels of models with an fp32 residual stream, softmax
attention, decayed linear attention, latent attention, gated linear recurrence.  Storage is bf16 or fp32, taken from the tensors; the
arithmetic is fp32."""
from __future__ import annotations

from dataclasses import dataclass
from typing import List, Optional, Sequence, Tuple

import torch

LC = 64                                     # tokens per chunk of the linear-attention kernel
ACTIVATIONS = {"silu": 1, "gelu_tanh": 2, "relu2": 3}
_DECODE_COLUMNS = (1, 2, 3, 4, 6, 8, 12, 16)   # latent widths, in units of 32, the matrix-core decode kernel is built for


@dataclass
class TokenBatch:
    """Tokens of several sequences, packed one after the other.  `lens` / `past`: new and earlier tokens per sequence (host); `cu` [B + 1]
    int32, `seq` [M] int32, `pos` [M] int64, `resume` [B] int32 (sequences that go on from a cached state): on the device.  A decode step
    (`decode`: one token per cache row, positions known to the device only) has no host lengths."""
    cu: Optional[torch.Tensor]
    seq: Optional[torch.Tensor]
    pos: torch.Tensor
    resume: Optional[torch.Tensor]
    lens: List[int]
    past: List[int]
    decode: bool = False

    @staticmethod
    def of_prompts(lens: Sequence[int], past: Sequence[int], device) -> "TokenBatch":
        lens, past = list(lens), list(past)
        B, M, device = len(lens), sum(lens), torch.device(device)
        host = torch.tensor([[0] + lens, [0] + past], dtype=torch.int64).to(device)       # (one copy; the rest is made on the device)
        cu = host[0].cumsum(0)
        seq = torch.repeat_interleave(torch.arange(B, device=device), host[0, 1:], output_size=M)
        pos = torch.arange(M, device=device) + (host[1, 1:] - cu[:-1])[seq]
        resume = (host[1, 1:] > 0).to(torch.int32) if any(past) else None
        return TokenBatch(cu.to(torch.int32), seq.to(torch.int32), pos, resume, lens, past)

    @staticmethod
    def of_decode(pos: torch.Tensor) -> "TokenBatch":
        return TokenBatch(None, None, pos, None, [], [], decode=True)


class Stream:
    """The fp32 residual stream x [M, D] of one pass, its storage-type copy, and at most one sublayer output that has not been added yet: for a
    few rows of bf16 the next layer's launch adds it (ops.postnorm_linear / postnorm_gate), otherwise it is added at once.

    The norm of a sublayer's output y comes before the addition, x <- x + norm(y), or -- with `alpha` -- behind it, x <- norm(alpha x + y);
    norm(t) = t / rms(t) * (w_offset + w)."""

    def __init__(self, ops, ids: torch.Tensor, weight: torch.Tensor, scale: float, eps: float, w_offset: float, alpha: Optional[float] = None):
        self.ops, self.eps, self.w_offset, self.alpha = ops, eps, w_offset, alpha
        self.x, self.xb = ops.embed_stream(ids, weight, scale)
        self.open = None                                         # (y, w): still to be added
        self.spare = None                                        # the buffer the next such launch writes x to
        self.behind = False                                      # xb does not hold the current x

    def add(self, y: torch.Tensor, w: torch.Tensor) -> None:
        self.flush()
        self.open = (y, w)
        if not self.ops.fuse_postnorm_ok(y):
            self.flush()

    def flush(self) -> None:
        if self.open is not None:
            y, w = self.open
            self.open = None
            if self.xb.dtype == self.x.dtype:
                self.xb = self.x
            if self.alpha is None:
                self.ops.postnorm_residual_(self.x, self.xb, y, w, self.eps, self.w_offset)
            else:
                self.ops.sum_norm_(self.x, self.xb, y, w, self.alpha, self.eps, self.w_offset)
            self.behind = False

    def input(self) -> torch.Tensor:
        """The sublayer input in the storage type."""
        self.flush()
        if self.behind:
            self.xb = self.x.to(self.xb.dtype)
            self.behind = False
        return self.xb

    def _swap(self):
        """(y, norm weight, x, where the new x goes) for a launch that adds the open output."""
        y, w = self.open
        self.open = None
        old, new = self.x, torch.empty_like(self.x) if self.spare is None else self.spare
        self.x, self.spare, self.behind = new, old, True
        return y, w, old, new

    def linear(self, w: torch.Tensor, act: Optional[str] = None) -> torch.Tensor:
        if self.open is None:
            return self.ops.linear(self.input(), w) if act is None else self.ops.linear_act(self.input(), w, act, w.shape[0])
        return self.ops.postnorm_linear(*self._swap(), w, self.eps, self.w_offset, alpha=self.alpha, act=act)

    def gate(self, w12: torch.Tensor, grouped: bool, act: str) -> torch.Tensor:
        if self.open is None:
            return self.ops.mlp_gate(self.input(), None if grouped else w12, w12g=w12 if grouped else None, act=act)
        return self.ops.postnorm_gate(*self._swap(), w12, grouped, act, self.eps, self.w_offset, alpha=self.alpha)

    def final(self, w: torch.Tensor) -> torch.Tensor:
        self.flush()
        return self.ops.rmsnorm_stream(self.x, w, self.eps, self.w_offset)


class MixerOps:
    """Mixed into HipOps (needs its `lib`, `_t`, `validate_ids`)."""

    mixer_mfma = True          # False: the any-size kernels in place of the matrix-core ones (tests, measurements)

    @staticmethod
    def _store(*tensors) -> int:
        """Checks one storage type on the device; 1 for fp32, 0 for bf16."""
        dt = tensors[0].dtype
        for t in tensors:
            if not t.is_cuda:
                raise RuntimeError(f"tensor is on {t.device}; the HIP path has no CPU fallback")
            if t.dtype != dt or dt not in (torch.float32, torch.bfloat16):
                raise RuntimeError(f"expected one storage type, fp32 or bf16, got {t.dtype} beside {dt}")
            if t.stride(-1) != 1:
                raise RuntimeError("tensor rows must be dense")
        return int(dt == torch.float32)

    @staticmethod
    def _ix(t: Optional[torch.Tensor], dtype, n: int, what: str) -> Optional[int]:
        if t is None:
            return None
        if not t.is_cuda or t.dtype != dtype or not t.is_contiguous() or t.numel() < n:
            raise RuntimeError(f"{what}: need a contiguous device {dtype} tensor of at least {n} entries")
        return t.data_ptr()

    @staticmethod
    def _dense(t: torch.Tensor, shape, what: str):
        if tuple(t.shape) != tuple(shape) or not t.is_contiguous():
            raise RuntimeError(f"{what}: need a contiguous tensor of shape {tuple(shape)}, got {tuple(t.shape)}")

    def _call(self, name: str, *args):
        from .ops import _check, _stream
        with self._t(name[4:]):
            _check(getattr(self.lib, name)(*args, _stream()), name)

    # ---- residual stream ------------------------------------------------------------------------------------------------
    def embed_stream(self, ids: torch.Tensor, weight: torch.Tensor, scale: float) -> Tuple[torch.Tensor, torch.Tensor]:
        """(x fp32 [M, D] = scale * weight[ids], the same in the storage type: x itself for fp32)."""
        ids = ids.reshape(-1).to(torch.int64).contiguous()
        f32 = self._store(weight)
        V, D = weight.shape
        self._dense(weight, (V, D), "embedding table")
        x = torch.empty(ids.numel(), D, dtype=torch.float32, device=weight.device)
        xb = x if f32 else torch.empty(ids.numel(), D, dtype=torch.bfloat16, device=weight.device)
        flag = None if torch.cuda.is_current_stream_capturing() or not self.validate_ids else \
            torch.zeros(1, dtype=torch.int32, device=weight.device)
        self._call("evo_embed_stream", self._ix(ids, torch.int64, ids.numel(), "ids"), weight.data_ptr(), x.data_ptr(), None if f32 else xb.data_ptr(),
                   ids.numel(), D, V, float(scale), None if flag is None else flag.data_ptr(), f32)
        if flag is not None and int(flag.item()) != 0:
            raise IndexError(f"input_ids contain values outside [0, {V}) (embedding table has {V} rows)")
        return x, xb

    def _closing_args(self, x, xb, y, w):
        f32 = self._store(y, w, xb)
        M, D = y.shape
        self._dense(y, (M, D), "y"), self._dense(x, (M, D), "x"), self._dense(xb, (M, D), "xb"), self._dense(w, (D,), "w")
        assert x.dtype == torch.float32 and (not f32 or xb is x)
        return y.data_ptr(), w.data_ptr(), x.data_ptr(), None if f32 else xb.data_ptr(), M, D

    def postnorm_residual_(self, x: torch.Tensor, xb: torch.Tensor, y: torch.Tensor, w: torch.Tensor, eps: float, w_offset: float) -> None:
        """x += rms_norm(y) * (w_offset + w) in place; xb (the storage-type copy of x, or x itself) follows."""
        self._call("evo_postnorm_residual", *self._closing_args(x, xb, y, w), float(eps), float(w_offset), int(y.dtype == torch.float32))

    def sum_norm_(self, x: torch.Tensor, xb: torch.Tensor, y: torch.Tensor, w: torch.Tensor, alpha: float, eps: float, w_offset: float) -> None:
        """x = rms_norm(alpha x + y) * (w_offset + w) in place; xb follows."""
        self._call("evo_sum_norm", *self._closing_args(x, xb, y, w), float(alpha), float(eps), float(w_offset), int(y.dtype == torch.float32))

    fuse_postnorm = True       # False: every closing norm as its own launch (tests, measurements)

    def fuse_postnorm_ok(self, y: torch.Tensor) -> bool:
        M, D = y.shape
        return self.fuse_postnorm and y.dtype == torch.bfloat16 and M <= 4 and D % 8 == 0 and D <= 8192

    def _postnorm_args(self, y, g, x, x_out, w):
        M, K = y.shape
        assert self._store(y, g, w) == 0
        for t, shape, what in ((y, (M, K), "y"), (g, (K,), "g"), (x, (M, K), "x"), (x_out, (M, K), "x_out"), (w, (w.shape[0], K), "w")):
            self._dense(t, shape, what)
        assert x.dtype == torch.float32 and x_out.dtype == torch.float32 and x.data_ptr() != x_out.data_ptr()
        return y.data_ptr(), g.data_ptr(), x.data_ptr(), x_out.data_ptr(), w.data_ptr()

    def postnorm_linear(self, y, g, x, x_out, w, eps: float, w_offset: float, alpha: Optional[float] = None, act: Optional[str] = None) -> torch.Tensor:
        """x_out = x + norm(y) * (w_offset + g), or norm(alpha x + y) * (w_offset + g); -> act(x_out @ w^T), one launch for up to four rows."""
        M, K = y.shape
        z = torch.empty(M, w.shape[0], dtype=y.dtype, device=y.device)
        fused = act in (None, "relu2")
        self._call("evo_postnorm_linear_small_m_bf16", *self._postnorm_args(y, g, x, x_out, w), z.data_ptr(), M, w.shape[0], K, float(alpha or 0.0),
                   int(alpha is not None), float(eps), float(w_offset), ACTIVATIONS[act] if fused and act else 0)
        if not fused:
            self.act_cols_(z, z.shape[1], act)
        return z

    def postnorm_gate(self, y, g, x, x_out, w12, grouped: bool, act: str, eps: float, w_offset: float, alpha: Optional[float] = None) -> torch.Tensor:
        """x_out as above; -> the gated MLP's first half on it, in the same launch."""
        M, K = y.shape
        I = w12.shape[0] // 2
        a = torch.empty(M, I, dtype=y.dtype, device=y.device)
        self._call("evo_postnorm_mlp_gate_small_m_bf16", *self._postnorm_args(y, g, x, x_out, w12), a.data_ptr(), M, I, K, float(alpha or 0.0),
                   int(alpha is not None), float(eps), float(w_offset), int(grouped), {"gelu": 0, "silu": 1}[act])
        return a

    def rmsnorm_stream(self, x: torch.Tensor, w: torch.Tensor, eps: float, w_offset: float) -> torch.Tensor:
        f32 = self._store(w)
        M, D = x.shape
        self._dense(x, (M, D), "x"), self._dense(w, (D,), "w")
        assert x.dtype == torch.float32 and x.is_cuda
        out = torch.empty(M, D, dtype=w.dtype, device=x.device)
        self._call("evo_rmsnorm_stream", x.data_ptr(), w.data_ptr(), out.data_ptr(), M, D, float(eps), float(w_offset), f32)
        return out

    def gated_norm(self, o: torch.Tensor, g: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
        """rms_norm(o) * w * sigmoid(g); g [M, D] may be a column range of a wider matrix."""
        f32 = self._store(o, g, w)
        M, D = o.shape
        self._dense(o, (M, D), "o"), self._dense(w, (D,), "w")
        assert tuple(g.shape) == (M, D)
        out = torch.empty_like(o)
        self._call("evo_gated_norm", o.data_ptr(), g.data_ptr(), g.stride(0), w.data_ptr(), out.data_ptr(), M, D, float(eps), f32)
        return out

    def silu_gate(self, z: torch.Tensor) -> torch.Tensor:
        f32 = self._store(z)
        M, I2 = z.shape
        self._dense(z, (M, I2), "z")
        a = torch.empty(M, I2 // 2, dtype=z.dtype, device=z.device)
        self._call("evo_silu_gate", z.data_ptr(), a.data_ptr(), M, I2 // 2, f32)
        return a

    def linear_act(self, x: torch.Tensor, w: torch.Tensor, act: str, act_cols: int, b: Optional[torch.Tensor] = None) -> torch.Tensor:
        """x @ w^T (+ b) with an activation on the first `act_cols` columns; in the dense layer's epilogue for prefill-sized
        batches and, the square of relu on all columns, for decode-sized ones."""
        M, K = x.shape
        N = w.shape[0]
        if act == "relu2" and act_cols == N and self._use_small_m(x, w):
            return self._linear_small_m(x, w, b, None, act=ACTIVATIONS[act])
        if (self._take_mfma(False) and self.mfma_linear_ok(x, w) and not self._use_small_m(x, w) and act_cols % 256 == 0 and K >= 128
                and M * K * 2 < 0xffffffff and N * K * 2 < 0xffffffff):
            r = self._tail_rows(x, w)
            y = torch.empty(M, N, dtype=x.dtype, device=x.device)
            self._call("evo_linear_act_mfma_bf16", x.data_ptr(), w.data_ptr(), None if b is None else b.data_ptr(), y.data_ptr(), M - r, N, K, act_cols,
                       ACTIVATIONS[act])
            if r:
                self._linear_small_m(x[M - r:], w, b, None, out=y[M - r:])
                self.act_cols_(y[M - r:], act_cols, act)
            return y
        y = self.linear(x, w, b)
        self.act_cols_(y, act_cols, act)
        return y

    def act_cols_(self, z: torch.Tensor, n: int, act: str) -> None:
        """z[:, :n] = act(z[:, :n]) in place"""
        f32 = self._store(z)
        assert z.dim() == 2 and z.shape[1] >= n
        self._call("evo_act_cols", z.data_ptr(), z.stride(0), z.shape[0], n, ACTIVATIONS[act], f32)

    # ---- decayed linear attention ---------------------------------------------------------------------------------------
    def lightning(self, z: torch.Tensor, heads: int, dk: int, dv: int, decay: torch.Tensor, log2_decay: torch.Tensor, batch: TokenBatch,
                  state: Optional[torch.Tensor] = None, seg_len: Optional[int] = None) -> torch.Tensor:
        """z [M, >= heads (2 dk + dv)] = [q | k | v | ..] -> o [M, heads dv]: after their SiLU for prompts (linear_act), before it for a decode
        step (the step applies it).  `state` [rows, heads, dk, dv] fp32 follows."""
        f32 = self._store(z)
        M = z.shape[0]
        o = torch.empty(M, heads * dv, dtype=z.dtype, device=z.device)
        assert z.shape[1] >= heads * (2 * dk + dv) and decay.numel() == heads and log2_decay.numel() == heads
        B = M if batch.decode else len(batch.lens)
        if state is not None:
            self._dense(state, (state.shape[0], heads, dk, dv), "state")
            assert state.dtype == torch.float32 and state.is_cuda and state.shape[0] >= B
        sp = None if state is None else state.data_ptr()
        dp = self._ix(decay, torch.float32, heads, "decay")
        if batch.decode:
            self._call("evo_lightning_recurrent", z.data_ptr(), z.stride(0), o.data_ptr(), sp, dp, None, None, B, heads, dk, dv, 1, f32)
            return o
        assert sum(batch.lens) == M
        cu, resume = self._ix(batch.cu, torch.int32, B + 1, "cu"), self._ix(batch.resume, torch.int32, B, "resume")
        if f32 or dk > 128 or not self.mixer_mfma:
            self._call("evo_lightning_recurrent", z.data_ptr(), z.stride(0), o.data_ptr(), sp, dp, cu, resume, B, heads, dk, dv, 0, f32)
            return o
        L = max(batch.lens)
        seg_len = seg_len or self.lightning_segment(L, B * heads * ((dv + 127) // 128))
        n_seg = (L + seg_len - 1) // seg_len
        seg = torch.empty(B, n_seg, heads, dk, dv, dtype=torch.float32, device=z.device) if n_seg > 1 else None
        self._call("evo_lightning_chunk_bf16", z.data_ptr(), z.stride(0), o.data_ptr(), sp, None if seg is None else seg.data_ptr(),
                   self._ix(log2_decay, torch.float32, heads, "log2_decay"), cu, resume, B, heads, dk, dv, L, seg_len)
        return o

    @staticmethod
    def lightning_segment(L: int, columns: int, target: int = 256) -> int:
        """Tokens per segment: one segment when (sequence, head) pairs alone fill the chip, else enough segments for a workgroup per CU,
        of at least four chunks each (a segment's state costs as much traffic as ~dk + dv tokens)."""
        want = max(1, (target + columns - 1) // columns)
        return max(4 * LC, (L + want * LC - 1) // (want * LC) * LC)

    # ---- latent attention -----------------------------------------------------------------------------------------------
    @staticmethod
    def latent_row(R: int, dr: int) -> int:
        """Elements of a cached row [latent | rotated key | zeros]: whole 32-wide steps, one or two more than a latent width the matrix-core
        decode kernel is built for, where the rotated part allows it."""
        need = (R + dr + 31) // 32
        fit = [max(need, c + 1) for c in _DECODE_COLUMNS if c * 32 >= R and need <= c + 2]
        return 32 * (min(fit) if fit else need)

    def latent_prep(self, qd: torch.Tensor, heads: int, dn: int, dr: int, R: int, norm_w: torch.Tensor, inv_freq: torch.Tensor, eps: float,
                    batch: TokenBatch, cache: Optional[torch.Tensor], want_kv: bool):
        """Rotates qd's query part in place; -> (c [M, R], kr [M, dr]) with `want_kv`; appends to the ring cache [rows, ring, row]."""
        f32 = self._store(qd, norm_w) if cache is None else self._store(qd, norm_w, cache)
        M = qd.shape[0]
        c = torch.empty(M, R, dtype=qd.dtype, device=qd.device) if want_kv else None
        kr = torch.empty(M, dr, dtype=qd.dtype, device=qd.device) if want_kv else None
        assert qd.shape[1] >= heads * (dn + dr) + R + dr and norm_w.numel() == R
        B = M if batch.decode else len(batch.lens)
        ring = rs = 0
        if cache is not None:
            rows, ring, rs = cache.shape
            self._dense(cache, (rows, ring, rs), "latent cache")
            assert rows >= B
        self._call("evo_latent_prep", qd.data_ptr(), qd.stride(0), None if c is None else c.data_ptr(), None if kr is None else kr.data_ptr(),
                   None if cache is None else cache.data_ptr(), norm_w.data_ptr(), self._ix(inv_freq, torch.float32, 0, "inv_freq"),
                   self._ix(batch.pos, torch.int64, M, "pos"), self._ix(batch.seq, torch.int32, M, "seq"),
                   self._ix(batch.cu, torch.int32, B + 1, "cu"), M, heads, dn, dr, R, 2 * inv_freq.numel(), ring, rs, float(eps), f32)
        return c, kr

    def window_attention(self, qd: torch.Tensor, kv: torch.Tensor, kr: torch.Tensor, heads: int, dn: int, dr: int, dv: int, window: int,
                         scale: float, sink: torch.Tensor, cu_q: torch.Tensor, cu_k: torch.Tensor, max_q: int) -> torch.Tensor:
        """qd rows start with the heads' [dn | dr] queries; kv rows = [keys (heads dn) | values (heads dv)]; kr [Mk, dr] -> [Mq, heads dv]."""
        nk = heads * dn
        assert kv.shape[1] == heads * (dn + dv) and kr.shape == (kv.shape[0], dr) and kr.is_contiguous() and kr.dtype == qd.dtype
        assert sink.numel() == heads and qd.shape[1] >= heads * (dn + dr)
        return self._window_attn(qd, kv[:, :nk], kv[:, nk:], kr, sink, heads, heads, 1, dn, dr, dv, window, 0, scale, 0.0, 1.0, 0.0, cu_q, cu_k, max_q)

    def _window_attn(self, q, kn, v, kr, sink, heads, kv_heads, maps, dn, dr, dv, window, keep, scale, lam, gain, eps, cu_q, cu_k, max_q):
        f32 = self._store(q, kn, v)
        B = cu_q.numel() - 1
        assert cu_k.numel() == B + 1 and kn.stride(0) == v.stride(0)
        o = torch.empty(q.shape[0], heads * dv, dtype=q.dtype, device=q.device)
        self._call("evo_window_attn", q.data_ptr(), q.stride(0), kn.data_ptr(), v.data_ptr(), kn.stride(0), None if kr is None else kr.data_ptr(),
                   o.data_ptr(), self._ix(cu_q, torch.int32, B + 1, "cu_q"), self._ix(cu_k, torch.int32, B + 1, "cu_k"),
                   self._ix(sink, torch.float32, heads, "sink"), B, heads, kv_heads, maps, dn, dr, dv, int(min(window, 1 << 29)), int(keep), int(max_q),
                   float(scale), float(lam), float(gain), float(eps), f32, int(self.mixer_mfma))
        return o

    @staticmethod
    def latent_split(B: int, heads: int, tiles: int, cus: int = 256):
        """(parts of the window, heads per workgroup) of the decode kernel: a workgroup per CU.  16 heads per workgroup get through a tile
        quicker, 32 read it once for twice the heads: the former while that leaves a workgroup at most four tiles."""
        def parts(groups):
            return max(1, min(tiles, cus // (B * groups), 32))
        n = parts((heads + 15) // 16)
        if (tiles + n - 1) // n <= 4 or heads <= 16:
            return n, 16
        return parts((heads + 31) // 32), 32

    def latent_decode(self, qd: torch.Tensor, cache: torch.Tensor, pos: torch.Tensor, wuk: torch.Tensor, wuv: torch.Tensor, sink: torch.Tensor,
                      heads: int, dn: int, dr: int, dv: int, R: int, window: int, scale: float, n_split: Optional[int] = None) -> torch.Tensor:
        """One token per cache row (already appended by latent_prep) against the ring cache -> [B, heads dv]."""
        f32 = self._store(qd, cache, wuk, wuv)
        B = qd.shape[0]
        rows, ring, rs = cache.shape
        self._dense(cache, (rows, ring, rs), "latent cache")
        self._dense(wuk, (heads * dn, R), "wuk"), self._dense(wuv, (heads * dv, R), "wuv")
        assert rows >= B and qd.shape[1] >= heads * (dn + dr) and window <= ring and sink.numel() == heads
        q = torch.empty(B, heads, rs, dtype=qd.dtype, device=qd.device)
        self._call("evo_latent_absorb", qd.data_ptr(), qd.stride(0), wuk.data_ptr(), q.data_ptr(), B, heads, dn, dr, R, rs, f32)
        group = 1
        if n_split is None:
            n_split, group = self.latent_split(B, heads, (ring + 63) // 64)
        part_o = torch.empty(B, heads, n_split, R, dtype=torch.float32, device=qd.device)
        part_ml = torch.empty(B, heads, n_split, 2, dtype=torch.float32, device=qd.device)
        self._call("evo_latent_decode", q.data_ptr(), cache.data_ptr(), self._ix(pos, torch.int64, B, "pos"), part_o.data_ptr(), part_ml.data_ptr(),
                   B, heads, R, dr, rs, ring, int(window), n_split, float(scale), f32, group if self.mixer_mfma else 0)
        o = torch.empty(B, heads * dv, dtype=qd.dtype, device=qd.device)
        self._call("evo_latent_up", part_o.data_ptr(), part_ml.data_ptr(), self._ix(sink, torch.float32, heads, "sink"), wuv.data_ptr(), o.data_ptr(),
                   B, heads, R, dv, n_split, f32, int(self.mixer_mfma))
        return o

    # ---- attention with cached keys and values ---------------------------------------------------------------------------
    def heads_prep(self, z: torch.Tensor, nq: int, nk: int, dim: int, nv: int, qk_norm, inv_freq: torch.Tensor, amp: float, unit: bool, eps: float,
                   batch: TokenBatch, cache: Optional[torch.Tensor], keep: int) -> None:
        """z rows = [nq query vectors | nk key vectors | nv values]: norms (`qk_norm`: (query weight, key weight) or None; `unit`: behind the
        rotation, without a weight) and rotation in place; keys and values go to the cache [rows, ring, row]."""
        f32 = self._store(z) if cache is None else self._store(z, cache)
        M, B = z.shape[0], z.shape[0] if batch.decode else len(batch.lens)
        assert z.shape[1] >= (nq + nk) * dim + nv
        qw, kw = qk_norm if qk_norm is not None else (None, None)
        for w in (qw, kw):
            if w is not None:
                self._store(z, w), self._dense(w, (dim,), "norm weight")
        ring = rs = 0
        if cache is not None:
            rows, ring, rs = cache.shape
            self._dense(cache, (rows, ring, rs), "key and value cache")
            assert rows >= B
        self._call("evo_heads_prep", z.data_ptr(), z.stride(0), None if cache is None else cache.data_ptr(), None if qw is None else qw.data_ptr(),
                   None if kw is None else kw.data_ptr(), self._ix(inv_freq, torch.float32, 0, "inv_freq"), self._ix(batch.pos, torch.int64, M, "pos"),
                   self._ix(batch.seq, torch.int32, M, "seq"), self._ix(batch.cu, torch.int32, B + 1, "cu"), M, nq, nk, dim, nv, 2 * inv_freq.numel(),
                   keep, ring, rs, float(amp), float(eps), int(unit), f32)

    def heads_attention(self, z: torch.Tensor, kv: torch.Tensor, heads: int, kv_heads: int, maps: int, dim: int, dv: int, window: Optional[int],
                        keep: int, scale: float, lam: float, gain: float, eps: float, cu_q: torch.Tensor, cu_k: torch.Tensor, max_q: int) -> torch.Tensor:
        """Queries at the start of z's rows against kv rows [keys | values] -> [Mq, heads dv]."""
        nk = kv_heads * maps * dim
        assert z.shape[1] >= heads * maps * dim and kv.shape[1] >= nk + kv_heads * dv
        return self._window_attn(z, kv[:, :nk], kv[:, nk:], None, None, heads, kv_heads, maps, dim, 0, dv, window or 1 << 29, keep, scale, lam, gain, eps,
                                 cu_q, cu_k, max_q)

    @staticmethod
    def heads_split(groups: int, ring: int, cus: int = 256) -> int:
        """Parts of the cache in the decode kernel: a workgroup per CU, at least 128 slots (one round of a workgroup's waves) each."""
        return max(1, min((ring + 127) // 128, (cus + groups - 1) // groups, 64))

    def heads_decode(self, z: torch.Tensor, cache: torch.Tensor, pos: torch.Tensor, heads: int, kv_heads: int, maps: int, dim: int, dv: int, scale: float,
                     lam: float, gain: float, eps: float, n_split: Optional[int] = None) -> torch.Tensor:
        """One token per cache row (already appended by heads_prep) -> [B, heads dv]."""
        f32 = self._store(z, cache)
        B = z.shape[0]
        rows, ring, rs = cache.shape
        self._dense(cache, (rows, ring, rs), "key and value cache")
        assert rows >= B and z.shape[1] >= heads * maps * dim and rs >= kv_heads * (maps * dim + dv)
        if n_split is None:
            n_split = self.heads_split(B * kv_heads * ((heads // kv_heads + 15) // 16), ring)
        part_o = torch.empty(B, heads * maps, n_split, dv, dtype=torch.float32, device=z.device)
        part_ml = torch.empty(B, heads * maps, n_split, 2, dtype=torch.float32, device=z.device)
        self._call("evo_heads_decode", z.data_ptr(), z.stride(0), cache.data_ptr(), self._ix(pos, torch.int64, B, "pos"), part_o.data_ptr(),
                   part_ml.data_ptr(), B, heads, kv_heads, maps, dim, dv, ring, rs, n_split, float(scale), f32, int(self.mixer_mfma))
        o = torch.empty(B, heads * dv, dtype=z.dtype, device=z.device)
        self._call("evo_heads_merge", part_o.data_ptr(), part_ml.data_ptr(), o.data_ptr(), B, heads, maps, dv, n_split, float(lam), float(gain), float(eps),
                   f32)
        return o

    # ---- gated linear recurrence ------------------------------------------------------------------------------------------
    @staticmethod
    def rglru_mfma_ok(W: int, blocks: int, taps: int, dtype) -> bool:
        bs = W // blocks
        return dtype == torch.bfloat16 and bs % 8 == 0 and bs <= 384 and taps <= 4

    @staticmethod
    def rglru_segment(L: int, walkers: int, target: int = 256) -> int:
        """Tokens per segment: one segment while the walking workgroups fill most of the chip, else as many as give every CU one (a segment's
        state costs another pass over its gates)."""
        want = max(1, target // walkers) if walkers <= target * 5 // 8 else 1
        return max(256, (L + want * 64 - 1) // (want * 64) * 64) if want > 1 else (L + 63) // 64 * 64

    def rglru(self, z: torch.Tensor, in_b: Optional[torch.Tensor], act: bool, W: int, conv: torch.Tensor, conv_b: torch.Tensor, ra, ra_b, ri, ri_b,
              decay: torch.Tensor, batch: TokenBatch, state: Optional[torch.Tensor] = None, seg_len: Optional[int] = None) -> torch.Tensor:
        """z [M, >= 2 W] = [y | x] -> o [M, W]; `in_b` [2 W]: still to be added to z; `act`: y is before its activation.  `state`
        [rows, 1 + taps, W] fp32 follows."""
        f32 = self._store(z, conv, conv_b, ra, ra_b, ri, ri_b)
        M, nb, taps = z.shape[0], ra.shape[0], conv.shape[1]
        bs = W // nb
        for t, shape, what in ((conv, (W, taps), "conv"), (conv_b, (W,), "conv_b"), (ra, (nb, bs, bs), "ra"), (ri, (nb, bs, bs), "ri"), (ra_b, (nb, bs), "ra_b"),
                               (ri_b, (nb, bs), "ri_b")):
            self._dense(t, shape, what)
        assert z.shape[1] >= 2 * W and (in_b is None or (in_b.dtype == z.dtype and in_b.is_contiguous() and in_b.numel() >= 2 * W))
        B = M if batch.decode else len(batch.lens)
        if state is not None:
            self._dense(state, (state.shape[0], 1 + taps, W), "state")
            assert state.dtype == torch.float32 and state.is_cuda and state.shape[0] >= B
        o = torch.empty(M, W, dtype=z.dtype, device=z.device)
        head = (z.data_ptr(), z.stride(0))
        sp, bp = None if state is None else state.data_ptr(), None if in_b is None else in_b.data_ptr()
        w = (conv.data_ptr(), conv_b.data_ptr(), ra.data_ptr(), ra_b.data_ptr(), ri.data_ptr(), ri_b.data_ptr(), self._ix(decay, torch.float32, W, "decay"),
             self._ix(batch.pos, torch.int64, M, "pos"))
        fast = self.mixer_mfma and self.rglru_mfma_ok(W, nb, taps, z.dtype) and z.stride(0) % 8 == 0
        if batch.decode and fast:
            self._call("evo_rglru_step_bf16", *head, bp, o.data_ptr(), sp, *w, B, W, nb, taps, int(act))
            return o
        cu, resume = self._ix(batch.cu, torch.int32, B + 1, "cu"), self._ix(batch.resume, torch.int32, B, "resume")
        if fast and in_b is None and not act:
            assert sum(batch.lens) == M
            L = max(batch.lens)
            seg_len = seg_len or self.rglru_segment(L, B * nb * ((bs + 127) // 128))
            n_seg = (L + seg_len - 1) // seg_len
            seg = torch.empty(B, n_seg, 2, W, dtype=torch.float32, device=z.device) if n_seg > 1 else None
            self._call("evo_rglru_chunk_bf16", *head, o.data_ptr(), sp, None if seg is None else seg.data_ptr(), *w, cu, resume, B, W, nb, taps, L, seg_len)
            return o
        ab = torch.empty(M, 2, W, dtype=torch.float32, device=z.device)
        self._call("evo_rglru_any", *head, bp, o.data_ptr(), sp, ab.data_ptr(), *w, self._ix(batch.seq, torch.int32, M, "seq"), cu, resume, M, B, W, nb, taps,
                   int(act), f32)
        return o
