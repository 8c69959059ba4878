"""Decoders that a config.json describes layer by layer: an fp32 residual stream, a list of layers -- each a token mixer and a feed-forward or
none (evo_amd/mixers.py) --, a norm at every sublayer's end, a final norm and a head.

`LayeredDecoder` is everything such models share; a model class names its sublayer kinds (`MIXERS`, `FEED_FORWARDS`), how its norms store their
weight (`NORM_OFFSET`) and reads its own constants from the config.  It keeps the contract of evo_amd.sh.model.StripedHyena:
`model(ids, inference_params_dict)`, the two cache records, `hidden_states`, `unembed`, cache rows for the decode pool, the captured decode step.
It runs in bf16 (products and activations; everything that feeds a softmax, a norm, a recurrence or the stream in fp32) or, with
`dtype=torch.float32`, in fp32 throughout.  All arithmetic is dispatched to an `ops` object, as there; there is no CPU fallback.

A layer whose entry says `weights_of: j` runs layer j's sublayers once more, with a cache of its own.
"""
from __future__ import annotations

from typing import Dict, List, Optional

import torch
import torch.nn as nn

from .mixer_ops import Stream, TokenBatch
from .mixers import build_feed_forward, build_mixer
from .sh.cache import InferenceParams, RecurrentInferenceParams
from .sh.graph import DecodeGraphMixin
from .sh.utils import dotdict


class _Layer(nn.Module):
    def __init__(self, cfg, mixers, feed_forwards, width, eps, dtype, where):
        super().__init__()
        self.mix = build_mixer(mixers, cfg, width, eps, dtype, where)
        self.mlp = build_feed_forward(feed_forwards, cfg, width, dtype, where)


class _Head(nn.Module):
    weight: torch.Tensor


class LayeredDecoder(DecodeGraphMixin, nn.Module):
    MIXERS: dict = {}                    # config `type` / `kind` -> sublayer
    FEED_FORWARDS: dict = {}
    REQUIRED = ("vocab", "width", "layers", "norm")
    NORM_OFFSET = 0.0                    # norm(t) = t / rms(t) * (NORM_OFFSET + weight)
    embed_scale = 1.0
    alpha: Optional[float] = None        # None: x + norm(y); a number: norm(alpha x + y)   (mixer_ops.Stream)

    packs_prompts = True                 # prefill_rows runs unequal prompts as one pass
    spare_positions = 1024               # room for new tokens in caches that grow with the sequence
    max_rows_per_pass = 128 * 1024       # tokens of one packed prompt pass (prefill_rows); more prompts run in groups

    def __init__(self, config, ops=None, dtype: torch.dtype = torch.bfloat16):
        super().__init__()
        if not isinstance(config, dict):
            raise TypeError("config must be a dict / dotdict")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"dtype must be bfloat16 or float32, got {dtype}")
        self.config = config if isinstance(config, dotdict) else dotdict(config)
        c = self.config
        missing = [k for k in self.REQUIRED if c.get(k) is None]
        if missing:
            raise ValueError(f"config: {', '.join(missing)} missing")
        self.dtype = dtype
        self.vocab_size, self.hidden_size, self.num_layers = int(c["vocab"]), int(c["width"]), len(c["layers"])
        self.eps = float(c["norm"]["eps"])
        self.max_seqlen = int(c.get("max_seqlen") or 1 << 20)
        self._read_config(c)
        self.weights_of = [self._weights_of(i) for i in range(self.num_layers)]
        built = {i: _Layer(c["layers"][i], self.MIXERS, self.FEED_FORWARDS, self.hidden_size, self.eps, dtype, f"layers[{i}]")
                 for i in sorted(set(self.weights_of))}
        self.layers = nn.ModuleList(built[j] for j in self.weights_of)
        self.unembed = _Head()
        self._ops = ops
        self._loaded = False

    def _read_config(self, c) -> None:
        """The constants of a model class of its own."""

    def _weights_of(self, i: int) -> int:
        """The layer whose tensors layer i uses."""
        layers, j = self.config["layers"], i
        while layers[j].get("weights_of") is not None:
            k = int(layers[j]["weights_of"])
            if not 0 <= k < len(layers) or k == i or any(layers[k].get(x) != layers[i].get(x) for x in ("type", "mixer", "mlp")):
                raise ValueError(f"layers[{i}]: 'weights_of' must name another layer of the same kind and sizes")
            j = k
        return j

    def _own_layers(self):
        return [(i, self.layers[i]) for i in sorted(set(self.weights_of))]

    # ------------------------------------------------------------------ weights
    def tensor_shapes(self) -> Dict[str, tuple]:
        """{checkpoint tensor: shape}"""
        D, V = self.hidden_size, self.vocab_size
        out = {"embed": (V, D)}
        for i, layer in self._own_layers():
            out[f"l{i}.norm1"] = (D,)
            out.update({f"l{i}.mix.{k}": s for k, s in layer.mix.tensors().items()})
            if layer.mlp is not None:
                out[f"l{i}.norm2"] = (D,)
                out.update({f"l{i}.mlp.{k}": s for k, s in layer.mlp.tensors().items()})
        out.update({"final.norm": (D,), "head": (V, D)})
        return out

    def load_state_dict(self, state_dict, strict: bool = True, assign: bool = True):
        shapes = self.tensor_shapes()
        missing = [k for k in shapes if k not in state_dict]
        unexpected = [k for k in state_dict if k not in shapes]
        if missing or (strict and unexpected):
            raise RuntimeError(f"Error(s) in loading state_dict for {type(self).__name__}: missing keys {missing}, unexpected keys {unexpected}")
        for k, s in shapes.items():
            if tuple(state_dict[k].shape) != s:
                raise RuntimeError(f"size mismatch for {k}: checkpoint {tuple(state_dict[k].shape)} vs model {s}")

        def take(name):
            return state_dict[name].detach().to(self.dtype).contiguous()

        def below(prefix, names):
            return {k: state_dict[prefix + k] for k in names}
        self.register_buffer("embed", take("embed"), persistent=False)
        self.register_buffer("final_norm", take("final.norm"), persistent=False)
        self.unembed.register_buffer("weight", take("head"), persistent=False)
        for i, layer in self._own_layers():
            layer.register_buffer("norm1", take(f"l{i}.norm1"), persistent=False)
            layer.mix.load(below(f"l{i}.mix.", layer.mix.tensors()))
            if layer.mlp is not None:
                layer.register_buffer("norm2", take(f"l{i}.norm2"), persistent=False)
                layer.mlp.load(below(f"l{i}.mlp.", layer.mlp.tensors()))
        self._loaded = True
        from torch.nn.modules.module import _IncompatibleKeys
        return _IncompatibleKeys(missing, unexpected)

    def state_dict(self, *args, **kwargs):
        out = {"embed": self.embed, "final.norm": self.final_norm, "head": self.unembed.weight}
        for i, layer in self._own_layers():
            out[f"l{i}.norm1"] = layer.norm1
            out.update({f"l{i}.mix.{k}": t for k, t in layer.mix._views().items()})
            if layer.mlp is not None:
                out[f"l{i}.norm2"] = layer.norm2
                out.update({f"l{i}.mlp.{k}": t for k, t in layer.mlp._views().items()})
        return {k: out[k] for k in self.tensor_shapes()}

    def _apply(self, fn, recurse=True):
        out = super()._apply(fn, recurse)
        self.release_decode_graph()
        return out

    @property
    def device(self):
        return self.embed.device if self._loaded else torch.device("cpu")

    @property
    def ops(self):
        if self._ops is None:
            from .ops import default_ops
            self._ops = default_ops()          # raises if the HIP library / GPU is unavailable
        return self._ops

    # ------------------------------------------------------------------ caches
    def initialize_inference_params(self):
        """The records evo's generation loop reads and steps: "mha" holds the attention caches, "hyena" the recurrent states."""
        return {"mha": InferenceParams(max_seqlen=self.max_seqlen, max_batch_size=1, seqlen_offset=0),
                "hyena": RecurrentInferenceParams(seqlen_offset=0)}

    def allocate_rows(self, n_rows: int, capacity: int, old: Optional[dict] = None) -> dict:
        """State of `n_rows` independent sequences of up to `capacity` tokens; `old`: records whose rows are kept."""
        ipd = self.initialize_inference_params()
        ipd["mha"].max_batch_size = ipd["hyena"].max_batch_size = n_rows
        for i, layer in enumerate(self.layers):
            t = layer.mix.new_cache(n_rows, self.device, capacity)
            if old is not None:
                prev = layer.mix.store(old)[i]
                t[: prev.shape[0], : prev.shape[1]] = prev
            layer.mix.store(ipd)[i] = t
        return ipd

    def copy_row(self, dst: dict, dst_row: int, src: dict, src_row: int, n_tokens: int) -> None:
        """One sequence's state after `n_tokens` tokens from one set of rows to another."""
        for i, layer in enumerate(self.layers):
            d, s = layer.mix.store(dst)[i][dst_row], layer.mix.store(src)[i][src_row]
            if layer.mix.grows:
                d, s = d[:n_tokens], s[:n_tokens]
            d.copy_(s)

    def _room(self, ipd) -> int:
        """Positions the records hold."""
        return min((layer.mix.store(ipd)[i].shape[1] for i, layer in enumerate(self.layers) if layer.mix.grows), default=1 << 62)

    def _grow(self, ipd, need: int) -> None:
        """More positions in the caches that grow with the sequence, at least `need` and at least twice as many."""
        for i, layer in enumerate(self.layers):
            if layer.mix.grows:
                old = layer.mix.store(ipd)[i]
                new = layer.mix.new_cache(old.shape[0], old.device, max(need + self.spare_positions, 2 * old.shape[1]))
                new[:, : old.shape[1]] = old
                layer.mix.store(ipd)[i] = new

    def prefill_rows(self, prompts: List[torch.Tensor], want: Optional[List[List[int]]] = None):
        """Prompts of any lengths as packed passes -> [(logits [wanted, V], records, row of the records)]; `want`: the places whose logits are
        returned (the last token's by default)."""
        out, first = [], 0
        while first < len(prompts):
            n, tokens = 0, 0
            while first + n < len(prompts) and (n == 0 or tokens + prompts[first + n].numel() <= self.max_rows_per_pass):
                tokens += prompts[first + n].numel()
                n += 1
            group = prompts[first:first + n]
            lens = [p.numel() for p in group]
            ipd = self.allocate_rows(n, max(lens))
            h = self._run(torch.cat([p.reshape(-1) for p in group]), TokenBatch.of_prompts(lens, [0] * n, self.device), ipd)
            at = [[m - 1] for m in lens] if want is None else want[first:first + n]
            base = [sum(lens[:i]) for i in range(n)]
            rows = torch.tensor([b + t for b, ts in zip(base, at) for t in ts], dtype=torch.int64, device=h.device)
            logits = self.ops.linear(h[rows].contiguous(), self.unembed.weight) if rows.numel() else h.new_empty(0, self.vocab_size)
            out += [(lg, ipd, i) for i, lg in enumerate(logits.split([len(ts) for ts in at]))]
            first += n
        return out

    # ------------------------------------------------------------------ captured decode step (sh/graph.py)
    def _graph_tensors(self, ipd):
        out = {}
        for i, layer in enumerate(self.layers):
            store = layer.mix.store(ipd)
            if i not in store:
                return None
            out[i] = store[i]
        return out

    def _graph_room(self, ipd) -> int:
        return self._room(ipd)

    def _graph_grow(self, ipd, B: int, need: int) -> None:
        if need > self._room(ipd):
            self._grow(ipd, need)

    def _graph_shapes_ok(self, B: int) -> bool:
        """Every dense layer of a step of B rows takes the weight-streaming kernels: no library call is captured."""
        if self.dtype != torch.bfloat16 or not hasattr(self.ops, "small_m_shape_ok"):
            return False
        shapes = [tuple(self.unembed.weight.shape)]
        for layer in self.layers:
            shapes += layer.mix.dense_shapes() + ([] if layer.mlp is None else layer.mlp.dense_shapes())
        return all(self.ops.small_m_shape_ok(B, n, k) for n, k in shapes)

    # ------------------------------------------------------------------ forward
    def _run(self, ids: torch.Tensor, batch: TokenBatch, ipd: Optional[dict]) -> torch.Tensor:
        """Packed ids [M] -> final-norm hidden states [M, width] (logits = hidden @ head^T)."""
        if not self._loaded:
            raise RuntimeError(f"{type(self).__name__} has no weights: call load_state_dict first")
        ops = self.ops
        stream = Stream(ops, ids.to(self.device), self.embed, self.embed_scale, self.eps, self.NORM_OFFSET, self.alpha)
        taps = getattr(self, "block_taps", None)     # debugging / parity hook: residual stream entering every layer, then the final one
        for i, layer in enumerate(self.layers):
            if taps is not None:
                stream.flush()
                taps.append(stream.x.clone())
            stream.add(layer.mix.mix(ops, stream, batch, None if ipd is None else layer.mix.store(ipd)[i]), layer.norm1)
            if layer.mlp is not None:
                stream.add(layer.mlp.forward_ff(ops, stream), layer.norm2)
        if taps is not None:
            stream.flush()
            taps.append(stream.x.clone())
        return stream.final(self.final_norm)

    def hidden_states(self, x: torch.Tensor, inference_params_dict=None, padding_mask=None) -> torch.Tensor:
        """ids [B, T] -> final-norm hidden states [B T, width].  With records: the T tokens go on from `seqlen_offset`; one token per
        row at the rows' own positions when the KV record carries a `pos_tensor`."""
        if x.dim() != 2:
            raise ValueError("input_ids must be [batch, length]")
        if padding_mask is not None:
            raise ValueError(f"{type(self).__name__} takes no padding mask: unequal prompts are packed (prefill_rows), pads behind a prompt are never seen by it")
        B, T = x.shape
        if inference_params_dict is None:
            return self._run(x.reshape(-1), TokenBatch.of_prompts([T] * B, [0] * B, self.device), None)
        mha = inference_params_dict["mha"]
        pos = getattr(mha, "pos_tensor", None)
        off = int(mha.seqlen_offset)
        if pos is None and off > 0 and off + T > self._room(inference_params_dict):
            self._grow(inference_params_dict, off + T)
        if T == 1 and (pos is not None or off > 0):
            if pos is None:
                pos = torch.full((B,), off, dtype=torch.int64, device=self.device)
            return self._run(x.reshape(-1), TokenBatch.of_decode(pos), inference_params_dict)
        if off == 0:
            fresh = self.allocate_rows(max(B, int(mha.max_batch_size or 1)), T + self.spare_positions)
            for i, layer in enumerate(self.layers):
                layer.mix.store(inference_params_dict)[i] = layer.mix.store(fresh)[i]
        return self._run(x.reshape(-1), TokenBatch.of_prompts([T] * B, [off] * B, self.device), inference_params_dict)

    @torch.no_grad()
    def forward(self, x, inference_params_dict=None, padding_mask=None):
        """(logits [B, T, V] in the storage type, records or None)"""
        B, T = x.shape
        if T == 1 and inference_params_dict is not None and int(inference_params_dict["mha"].seqlen_offset) > 0 \
                and self._graph_eligible(inference_params_dict, B):
            logits = self._graph_decode_step(x, inference_params_dict)
            if logits is not None:
                return logits, inference_params_dict
        h = self.hidden_states(x, inference_params_dict, padding_mask)
        return self.ops.linear(h, self.unembed.weight).view(B, T, self.vocab_size), inference_params_dict
