"""TEST INFRASTRUCTURE: the mixer op set on the CPU, each op by the plain functions of oracle/{vozalorn,batodra}_ref.py.  It lets the host side of
evo_amd/decoder.py (packing, rings, slots, scheduling, generation) run in `-m "not gpu"` tests; the product never imports it.  On a model
with bf16 storage every op's result is rounded once: what rounding alone does to the logits, the yardstick of the bf16 GPU tests."""
import torch

from oracle import batodra_ref as R
from oracle import vozalorn_ref as V

ACT = {"silu": V.silu, "gelu_tanh": R.gelu_tanh, "relu2": R.squared_relu}


class MixerOracleOps:
    name = "oracle-cpu"

    def linear(self, x, w, b=None, mfma=False):
        y = x.double() @ w.double().T
        return (y if b is None else y + b.double()).to(x.dtype)

    def linear_act(self, x, w, act, act_cols, b=None):
        y = x.double() @ w.double().T
        y = y if b is None else y + b.double()
        return torch.cat([ACT[act](y[:, :act_cols]), y[:, act_cols:]], 1).to(x.dtype)

    def mlp_gate(self, x, w12, norm_scale=None, eps=0.0, w12g=None, act="gelu"):
        assert act == "silu" and norm_scale is None
        if w12 is None:                                           # rows come as [32 of the gate | the same 32 of up] blocks
            w12 = w12g.view(-1, 2, 32, w12g.shape[1]).transpose(0, 1).reshape(w12g.shape)
        z = x.double() @ w12.double().T
        I = z.shape[1] // 2
        return (V.silu(z[:, :I]) * z[:, I:]).to(x.dtype)

    def embed_stream(self, ids, weight, scale):
        if int(ids.min()) < 0 or int(ids.max()) >= weight.shape[0]:
            raise IndexError("input_ids contain values outside the table")
        x = weight[ids.reshape(-1)].float() * scale
        return x, x if weight.dtype == torch.float32 else x.to(weight.dtype)

    def postnorm_residual_(self, x, xb, y, w, eps, w_offset):
        x += (V.rms_normalise(y.double(), eps) * (w_offset + w.double())).float()
        if xb is not x:
            xb.copy_(x)

    def sum_norm_(self, x, xb, y, w, alpha, eps, w_offset):
        x.copy_(R.norm_of_sum(x.double(), y.double(), alpha, w_offset + w.double(), eps))
        if xb is not x:
            xb.copy_(x)

    @staticmethod
    def _closed(y, g, x, eps, w_offset, alpha):
        if alpha is None:
            return x + (V.rms_normalise(y.double(), eps) * (w_offset + g.double())).float()
        return R.norm_of_sum(x.double(), y.double(), alpha, w_offset + g.double(), eps).float()

    def fuse_postnorm_ok(self, y):
        return y.shape[0] <= 4                                    # (any storage: the host side of the fused form runs here too)

    def postnorm_linear(self, y, g, x, x_out, w, eps, w_offset, alpha=None, act=None):
        x_out.copy_(self._closed(y, g, x, eps, w_offset, alpha))
        return self.linear(x_out.to(y.dtype), w) if act is None else self.linear_act(x_out.to(y.dtype), w, act, w.shape[0])

    def postnorm_gate(self, y, g, x, x_out, w12, grouped, act, eps, w_offset, alpha=None):
        x_out.copy_(self._closed(y, g, x, eps, w_offset, alpha))
        return self.mlp_gate(x_out.to(y.dtype), None if grouped else w12, w12g=w12 if grouped else None, act=act)

    def rmsnorm_stream(self, x, w, eps, w_offset):
        return (V.rms_normalise(x.double(), eps) * (w_offset + w.double())).to(w.dtype)

    def gated_norm(self, o, g, w, eps):
        return (V.plain_rms_norm(o.double(), w.double(), eps) * torch.sigmoid(g.double())).to(o.dtype)

    @staticmethod
    def _spans(batch, M):
        if batch.decode:
            return [(b, b + 1) for b in range(M)]
        cu = batch.cu.tolist()
        return list(zip(cu[:-1], cu[1:]))

    def lightning(self, z, heads, dk, dv, decay, log2_decay, batch, state=None):
        out = torch.empty(z.shape[0], heads * dv, dtype=z.dtype)
        for b, (i, j) in enumerate(self._spans(batch, z.shape[0])):
            a = V.silu(z[i:j].double()) if batch.decode else z[i:j].double()
            q, k, v = a[:, :heads * dk], a[:, heads * dk:2 * heads * dk], a[:, 2 * heads * dk:heads * (2 * dk + dv)]
            keep = batch.decode or (batch.resume is not None and int(batch.resume[b]))
            o, S = V.decayed_linear_attention(q.view(-1, heads, dk), k.view(-1, heads, dk), v.view(-1, heads, dv), decay.tolist(),
                                              state[b].double() if keep else None)
            out[i:j] = o.reshape(j - i, -1)
            if state is not None:
                state[b] = S
        return out

    def latent_prep(self, qd, heads, dn, dr, R, norm_w, inv_freq, eps, batch, cache, want_kv):
        M, nq, half = qd.shape[0], heads * (dn + dr), inv_freq.numel()
        ang = batch.pos.double()[:, None] * inv_freq.double()

        def turn(x):                                              # [M, ..., dr]
            a = ang.reshape([M] + [1] * (x.dim() - 2) + [half])
            u, v = x[..., :half], x[..., half:2 * half]
            return torch.cat([u * a.cos() - v * a.sin(), v * a.cos() + u * a.sin(), x[..., 2 * half:]], -1)
        q = qd[:, :nq].view(M, heads, dn + dr).double()
        q[..., dn:] = turn(q[..., dn:])
        qd[:, :nq] = q.reshape(M, nq)
        c = V.plain_rms_norm(qd[:, nq:nq + R].double(), norm_w.double(), eps).to(qd.dtype)
        kr = turn(qd[:, nq + R:nq + R + dr].double()).to(qd.dtype)
        if cache is not None:
            ring = cache.shape[1]
            for b, (i, j) in enumerate(self._spans(batch, M)):
                for t in range(max(i, j - ring), j):
                    cache[b, int(batch.pos[t]) % ring, :R + dr] = torch.cat([c[t], kr[t]])
        return (c, kr) if want_kv else (None, None)

    def window_attention(self, qd, kv, kr, heads, dn, dr, dv, window, scale, sink, cu_q, cu_k, max_q):
        out = torch.empty(qd.shape[0], heads * dv, dtype=qd.dtype)
        cq, ck = cu_q.tolist(), cu_k.tolist()
        for b in range(len(cq) - 1):
            q = qd[cq[b]:cq[b + 1], :heads * (dn + dr)].double().view(-1, heads, dn + dr)
            J = ck[b + 1] - ck[b]
            kn = kv[ck[b]:ck[b + 1], :heads * dn].double().view(J, heads, dn)
            v = kv[ck[b]:ck[b + 1], heads * dn:].double().view(J, heads, dv)
            k = torch.cat([kn, kr[ck[b]:ck[b + 1], None].double().expand(J, heads, dr)], -1)
            kp = torch.arange(J)
            out[cq[b]:cq[b + 1]] = V.windowed_sink_attention(q, k, v, scale, window, sink, kp[J - q.shape[0]:], kp).reshape(q.shape[0], -1)
        return out

    def latent_decode(self, qd, cache, pos, wuk, wuv, sink, heads, dn, dr, dv, R, window, scale, n_split=None):
        B, ring = qd.shape[0], cache.shape[1]
        out = torch.empty(B, heads * dv, dtype=qd.dtype)
        for b in range(B):
            p = int(pos[b])
            js = list(range(max(0, p - window + 1), p + 1))
            rows = cache[b, [j % ring for j in js]].double()
            c, kr = rows[:, :R], rows[:, R:R + dr]
            k = torch.cat([(c @ wuk.double().T).view(len(js), heads, dn), kr[:, None].expand(len(js), heads, dr)], -1)
            v = (c @ wuv.double().T).view(len(js), heads, dv)
            q = qd[b:b + 1, :heads * (dn + dr)].double().view(1, heads, dn + dr)
            out[b] = V.windowed_sink_attention(q, k, v, scale, window, sink, torch.tensor([p]), torch.tensor(js)).reshape(-1)
        return out

    def heads_prep(self, z, nq, nk, dim, nv, qk_norm, inv_freq, amp, unit, eps, batch, cache, keep):
        M, nqk = z.shape[0], (nq + nk) * dim
        x = z[:, :nqk].double().view(M, nq + nk, dim)
        if qk_norm is not None:
            x = torch.cat([R.rms_norm(x[:, :nq], qk_norm[0].double(), eps), R.rms_norm(x[:, nq:], qk_norm[1].double(), eps)], 1)
        x = R.rotate(x, batch.pos, inv_freq.double().tolist(), amp)
        if unit:
            x = R.unit_rms(x, eps)
        z[:, :nqk] = x.reshape(M, nqk)
        if cache is not None:
            w = cache.shape[1] - keep
            for b, (i, j) in enumerate(self._spans(batch, M)):
                for t in range(i, j):
                    p = int(batch.pos[t])
                    if p < keep or j - t <= w:
                        cache[b, p if p < keep else keep + (p - keep) % w, :nk * dim + nv] = z[t, nq * dim:nqk + nv]

    @staticmethod
    def _combine(q, k, v, heads, maps, scale, lam, gain, eps, mask):
        """q [Tq, heads maps, n], k [Tk, G maps, n], v [Tk, G, dv]"""
        if maps == 1:
            return R.softmax_attention(q, k, v, scale, mask)
        a1, a2 = (R.softmax_attention(q[:, i::2], k[:, i::2], v, scale, mask) for i in (0, 1))
        return gain * R.unit_rms(a1 - lam * a2, eps)

    def heads_attention(self, z, kv, heads, kv_heads, maps, dim, dv, window, keep, scale, lam, gain, eps, cu_q, cu_k, max_q):
        out = torch.empty(z.shape[0], heads * dv, dtype=z.dtype)
        cq, ck, nk = cu_q.tolist(), cu_k.tolist(), kv_heads * maps * dim
        for b in range(len(cq) - 1):
            q = z[cq[b]:cq[b + 1], :heads * maps * dim].double().view(-1, heads * maps, dim)
            k, v = kv[ck[b]:ck[b + 1], :nk].double().view(-1, kv_heads * maps, dim), kv[ck[b]:ck[b + 1], nk:nk + kv_heads * dv].double().view(-1, kv_heads, dv)
            at = torch.arange(k.shape[0])                        # (indexes among the given keys: only their order counts)
            o = self._combine(q, k, v, heads, maps, scale, lam, gain, eps, R.visible(at[-q.shape[0]:], at, window, keep))
            out[cq[b]:cq[b + 1]] = o.reshape(q.shape[0], -1)
        return out

    def heads_decode(self, z, cache, pos, heads, kv_heads, maps, dim, dv, scale, lam, gain, eps, n_split=None):
        B, nk = z.shape[0], kv_heads * maps * dim
        out = torch.empty(B, heads * dv, dtype=z.dtype)
        for b in range(B):
            rows = cache[b, :min(int(pos[b]) + 1, cache.shape[1])].double()
            k, v = rows[:, :nk].view(-1, kv_heads * maps, dim), rows[:, nk:nk + kv_heads * dv].view(-1, kv_heads, dv)
            q = z[b:b + 1, :heads * maps * dim].double().view(1, heads * maps, dim)
            out[b] = self._combine(q, k, v, heads, maps, scale, lam, gain, eps, torch.ones(1, len(rows), dtype=torch.bool)).reshape(-1)
        return out

    def rglru(self, z, in_b, act, W, conv, conv_b, ra, ra_b, ri, ri_b, decay, batch, state=None, seg_len=None):
        out, n = torch.empty(z.shape[0], W, dtype=z.dtype), conv.shape[1]
        lam = torch.log(torch.expm1(decay.double() / -8.0))
        for b, (i, j) in enumerate(self._spans(batch, z.shape[0])):
            yx = z[i:j, :2 * W].double()
            yx = yx if in_b is None else yx + in_b[:2 * W].double()
            y, x = (R.gelu_tanh(yx[:, :W]) if act else yx[:, :W]), yx[:, W:]
            keep, p0 = batch.decode or (batch.resume is not None and int(batch.resume[b])), int(batch.pos[i])
            before = torch.zeros(n - 1, W, dtype=torch.float64)
            for k in range(1, n):
                if keep and p0 - k >= 0:
                    before[n - 1 - k] = state[b, 1 + (p0 - k) % n]
            u, _ = R.causal_convolution(x, conv.double(), conv_b.double(), before)
            if z.dtype == torch.bfloat16:
                u = u.to(z.dtype).double()
            r, g = (torch.sigmoid(R.block_diagonal(u, m.double(), c.double())) for m, c in ((ra, ra_b), (ri, ri_b)))
            S, last = R.gated_linear_recurrence(u, r, g, lam, state[b, 0].double() if keep else None)
            out[i:j] = S * y
            if state is not None:
                state[b, 0] = last
                for t in range(max(i, j - n), j):
                    state[b, 1 + int(batch.pos[t]) % n] = x[t - i]
        return out
