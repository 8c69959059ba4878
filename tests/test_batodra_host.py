"""CPU: the host side of the Batodra model -- registry, loading, shared layers, packing, rings, growing caches, slots, scheduling, generation, trace
replay -- on an op set made of plain functions (tests/mixer_oracle_ops.py), against the plain reference run one sequence at a time."""
import io
import json
import math
import sys

import numpy as np
import pytest
import torch
from safetensors.torch import save_file

import batodra_util as U
from mixer_oracle_ops import MixerOracleOps
from oracle import batodra_ref as R

TOL = 3e-5


def cpu_model(name, seed=0):
    cfg = U.CONFIGS[name]
    w = U.weights(cfg, seed)
    return cfg, U.build(cfg, w, ops=MixerOracleOps()), U.reference(cfg, w)


# ------------------------------------------------------------------------------------------------ the reference itself
def test_recurrence_and_convolution_by_hand():
    u = torch.tensor([[2.0], [1.0]], dtype=torch.float64)
    r, i = torch.tensor([[0.5], [0.25]], dtype=torch.float64), torch.tensor([[1.0], [0.5]], dtype=torch.float64)
    lam = torch.tensor([0.3], dtype=torch.float64)
    S, last = R.gated_linear_recurrence(u, r, i, lam)
    sp = math.log(1 + math.exp(0.3))
    a1, a2 = math.exp(-8 * 0.5 * sp), math.exp(-8 * 0.25 * sp)
    s1 = math.sqrt(1 - a1 * a1) * 2.0
    s2 = a2 * s1 + math.sqrt(1 - a2 * a2) * 0.5
    assert torch.allclose(S.flatten(), torch.tensor([s1, s2], dtype=torch.float64)) and float(last[0]) == float(S[1, 0])
    x, taps = torch.tensor([[1.0], [2.0], [4.0]]), torch.tensor([[10.0, 100.0, 1000.0]])
    v, tail = R.causal_convolution(x, taps, torch.tensor([0.5]))
    assert v.flatten().tolist() == [1000.5, 2100.5, 4210.5] and tail.flatten().tolist() == [2.0, 4.0]


def test_visibility_by_hand():
    pos = torch.arange(9)
    m = R.visible(pos, pos, window=3, keep_first=2)
    for i in range(9):
        assert [j for j in range(9) if m[i, j]] == sorted({j for j in range(i + 1) if i - j < 3 or j < 2})
    assert bool((R.visible(pos, pos) == torch.tril(torch.ones(9, 9, dtype=torch.bool))).all())


def test_differential_attention_by_hand():
    """Equal scores: each map is the mean of the values; the difference is (1 - lambda) of it, normed to 1 - diff."""
    q = torch.zeros(3, 1, 4, dtype=torch.float64)
    v = torch.tensor([[[1.0, -1.0]], [[3.0, -3.0]], [[5.0, -5.0]]], dtype=torch.float64)
    pos = torch.arange(3)
    a = R.softmax_attention(q, q, v, 1.0, R.visible(pos, pos))
    assert a[:, 0, 0].tolist() == [1.0, 2.0, 3.0]
    o = R.difference_of_maps(a, a, 0.4, 0.2, 0.0)
    assert torch.allclose(o, 0.8 * torch.tensor([[[1.0, -1.0]]] * 3, dtype=torch.float64))
    w = {"lq1": torch.tensor([1.0, 2.0]), "lk1": torch.tensor([0.5, 0.25]), "lq2": torch.tensor([1.0, 0.0]), "lk2": torch.tensor([-1.0, 9.0])}
    assert abs(float(R.difference_weight(w, 0.3)) - (math.e - math.exp(-1.0) + 0.3)) < 1e-6


def test_yarn_frequencies():
    """Fast pairs keep their frequency, slow ones are divided by the factor; the product's table is the same."""
    from evo_amd.mixers import rotation
    s = dict(factor=4.0, original=256, fast=16.0, slow=1.0)
    base, dims = 10000.0, 64
    plain = R.rotation_frequencies(base, dims)
    f, amp = R.yarn(plain, base, dims, **s)
    assert abs(amp - (0.1 * math.log(4.0) + 1.0)) < 1e-15 and f[0] == plain[0] and abs(f[-1] - plain[-1] / 4.0) < 1e-18
    turns = [256 * x / (2 * math.pi) for x in plain]
    assert all(abs(f[i] - plain[i]) < 1e-12 for i in range(32) if turns[i] > 16 * 1.4) and all(abs(f[i] - plain[i] / 4) < 1e-12 for i in range(32) if turns[i] < 0.7)
    got, got_amp = rotation(dict(base=base, dims=dims, scaling=s), "rot")
    assert torch.equal(got, torch.tensor(f, dtype=torch.float64).float()) and got_amp == amp
    for odd in (dict(factor=1.0, original=8, fast=1.0, slow=1.0), dict(factor=2.5, original=3, fast=40.0, slow=0.01), dict(factor=8.0, original=100000, fast=2.0, slow=1.9)):
        for n in (2, 6, 32):
            assert torch.allclose(rotation(dict(base=500.0, dims=n, scaling=odd), "r")[0].double(), torch.tensor(R.yarn(R.rotation_frequencies(500.0, n), 500.0, n, **odd)[0], dtype=torch.float64), rtol=1e-6)


# ------------------------------------------------------------------------------------------------ configuration and loading
def test_registry_and_config_errors():
    from evo_amd.batodra import Batodra
    from evo_amd.models import architecture_of
    assert architecture_of({"architecture": "Batodra"}) is Batodra
    for broken in (lambda c: c["layers"][0].update(type="latent_attention"), lambda c: c["layers"][0]["mixer"].pop("scale"), lambda c: c.pop("postln_alpha"),
                   lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), lambda c: c["layers"][0]["mixer"].update(kv_heads=3),
                   lambda c: c["layers"][1]["mixer"].update(blocks=5), lambda c: c["layers"][2]["mixer"].pop("diff"), lambda c: c["layers"][2]["mlp"].update(kind="other"),
                   lambda c: c["layers"][3].update(weights_of=9), lambda c: c["layers"][3].update(weights_of=1), lambda c: c["layers"][0]["mixer"]["rot"].update(dims=64)):
        c = json.loads(json.dumps(U.CONFIGS["plain"]))
        Batodra(c)
        broken(c)
        with pytest.raises(ValueError):
            Batodra(c)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("name", sorted(U.CONFIGS))
def test_state_dict_round_trip(name, dtype):
    cfg = U.CONFIGS[name]
    w = U.weights(cfg)
    m = U.build(cfg, w, dtype=dtype)
    assert m.tensor_shapes() == U.shapes_of(cfg)
    sd = m.state_dict()
    assert set(sd) == set(w) and all(torch.equal(sd[k].float(), w[k].float()) for k in w)


def test_wide_feed_forward_is_padded():
    """An inner size beyond 1,024 that is no multiple of 256: zero rows and columns, the checkpoint's tensors come back."""
    cfg = U.config([U.recurrence(ff=1100)], width=64)
    w = U.weights(cfg)
    m = U.build(cfg, w, dtype=torch.bfloat16, ops=MixerOracleOps())
    assert tuple(m.layers[0].mlp.w_up.shape) == (1280, 64) and all(torch.equal(t, w[k]) for k, t in m.state_dict().items())
    ids = U.tokens(cfg, 9)
    assert U.rel_err(m(torch.tensor([ids]))[0][0], U.reference(cfg, w)(ids)) < 5e-2


def test_strict_loading():
    cfg = U.CONFIGS["plain"]
    w = U.weights(cfg)
    m = U.build(cfg, w)
    for change in (lambda d: d.pop("l2.mix.lq1"), lambda d: d.update({"l3.norm1": torch.zeros(160)}), lambda d: d.update({"l1.mix.ra": torch.zeros(3, 3, 3)})):
        d = dict(w)
        change(d)
        with pytest.raises(RuntimeError):
            m.load_state_dict(d)


def test_model_folder(tmp_path):
    from evo_amd.models import load_model_dir
    cfg = U.CONFIGS["order"]
    w = U.weights(cfg)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file(w, str(tmp_path / "model.safetensors"))
    m = load_model_dir(str(tmp_path), dtype=torch.float32)
    m._ops = MixerOracleOps()
    ids = U.tokens(cfg, 12)
    assert U.rel_err(m(torch.tensor([ids]))[0][0], U.reference(cfg, w)(ids)) < TOL
    assert load_model_dir(str(tmp_path), weights="synthetic", seed=3).state_dict()["embed"].shape == (cfg["vocab"], cfg["width"])


# ------------------------------------------------------------------------------------------------ prompts, portions, decoding
@pytest.mark.parametrize("name", sorted(U.CONFIGS))
def test_prompt_and_token_by_token(name):
    cfg, m, ref = cpu_model(name)
    ids = U.tokens(cfg, 45)
    taps = []
    want = ref(ids, taps=taps)
    m.block_taps = []
    assert U.rel_err(m(torch.tensor([ids]))[0][0], want) < TOL
    for got, t in zip(m.block_taps[1:], taps):                   # the stream behind every layer
        assert U.rel_err(got, t) < TOL
    m.block_taps = None
    ipd = m.initialize_inference_params()
    got = [m(torch.tensor([ids[:30]]), ipd)[0][0]]
    for t in range(30, 45):
        ipd["mha"].seqlen_offset = ipd["hyena"].seqlen_offset = t
        got.append(m(torch.tensor([ids[t:t + 1]]), ipd)[0][0])
    assert U.rel_err(torch.cat(got), want) < TOL


@pytest.mark.parametrize("name", ["plain", "order", "odd", "window_1"])
@pytest.mark.parametrize("cuts", [[2] * 15, [1, 29], [29, 1], [13, 2, 15], [7, 7, 7, 9]])
def test_portions(name, cuts):
    cfg, m, ref = cpu_model(name)
    ids = U.tokens(cfg, 30)
    ipd = m.initialize_inference_params()
    got, at = [], 0
    for n in cuts:
        ipd["mha"].seqlen_offset = ipd["hyena"].seqlen_offset = at
        got.append(m(torch.tensor([ids[at:at + n]]), ipd)[0][0])
        at += n
    assert U.rel_err(torch.cat(got), ref(ids)) < TOL


def test_caches_grow_with_the_sequence():
    cfg, m, ref = cpu_model("plain")
    m.spare_positions = 2
    ids = U.tokens(cfg, 40)
    ipd = m.initialize_inference_params()
    got = [m(torch.tensor([ids[:5]]), ipd)[0][0]]
    at = 5
    for n in [1] * 9 + [6] + [1] * 8 + [12]:
        ipd["mha"].seqlen_offset = ipd["hyena"].seqlen_offset = at
        got.append(m(torch.tensor([ids[at:at + n]]), ipd)[0][0])
        at += n
    assert at == 40 and U.rel_err(torch.cat(got), ref(ids)) < TOL


def test_a_key_that_stands_out_at_every_distance():
    """One token that takes most of the attention: inside and outside of the window, among the kept first tokens and just behind them."""
    for keep, window in ((0, 6), (3, 6), (9, 4)):
        cfg = U.config([U.windowed(window=window, keep=keep, dim=16, rot=16)])
        w = U.spiky(cfg, U.weights(cfg))
        m, ref = U.build(cfg, w, ops=MixerOracleOps()), U.reference(cfg, w)
        base = [t if t != 7 else 8 for t in U.tokens(cfg, 26)]
        blank = ref(base)
        for at in range(0, 14):
            ids = base[:at] + [7] + base[at + 1:]
            want = ref(ids)
            for i in range(at, 26):                               # the reference itself: the token shows exactly where it is visible
                seen = i - at < window or at < keep
                assert (float((want[i] - blank[i]).abs().max()) > 0.05) == seen or i == at
            ipd = m.initialize_inference_params()
            got = [m(torch.tensor([ids[:10]]), ipd)[0][0]]
            for t in range(10, 26):
                ipd["mha"].seqlen_offset = ipd["hyena"].seqlen_offset = t
                got.append(m(torch.tensor([ids[t:t + 1]]), ipd)[0][0])
            assert U.rel_err(torch.cat(got), want) < TOL


def test_equal_length_batch():
    cfg, m, ref = cpu_model("plain")
    rows = [U.tokens(cfg, 20, s) for s in range(3)]
    got = m(torch.tensor(rows))[0]
    for r, g in zip(rows, got):
        assert U.rel_err(g, ref(r)) < TOL


def pool_of(m, n_slots=2, **kw):
    from evo_amd.pool import DecodePool
    from evo_amd.tokenizer import CharLevelTokenizer
    return DecodePool(m, CharLevelTokenizer(m.vocab_size), n_slots=n_slots, **kw)


@pytest.mark.parametrize("name", ["plain", "order", "odd"])
def test_unequal_requests_and_reused_slots(name):
    """Three waves of unequal requests on the same slots; some end early; every logit equals the request's alone."""
    cfg, m, ref = cpu_model(name)
    pool = pool_of(m, n_slots=1)
    for wave, lens in enumerate([[1, 17, 6], [9], [3, 30]]):
        reqs = [U.tokens(cfg, n + 8, seed=10 * wave + i) for i, n in enumerate(lens)]
        wants = [ref(r) for r in reqs]
        slots, got = pool.admit([torch.tensor(r[:n]) for r, n in zip(reqs, lens)], [list(range(n)) for n in lens])
        assert len(set(slots)) == len(slots)
        for g, w, n in zip(got, wants, lens):
            assert U.rel_err(g, w[:n]) < TOL
        live = dict(enumerate(slots))
        for t in range(8):
            lg = pool.advance({s: reqs[i][lens[i] + t] for i, s in live.items()})
            for i, s in live.items():
                assert U.rel_err(lg[s][None], wants[i][lens[i] + t][None]) < TOL
            if t == 2 and len(live) > 1:
                pool.release(live.pop(0))
        for s in live.values():
            pool.release(s)
    assert sorted(pool.free) == list(range(pool.n_slots)) and pool.n_slots == 3


def test_pool_grows_while_requests_live():
    cfg, m, ref = cpu_model("order")
    pool = pool_of(m, n_slots=1)
    a, b = U.tokens(cfg, 40, 1), U.tokens(cfg, 12, 2)
    wa, wb = ref(a), ref(b)
    (sa,), _ = pool.admit([torch.tensor(a[:5])])
    for t in range(5, 9):
        pool.advance({sa: a[t]})
    (sb,), _ = pool.admit([torch.tensor(b[:6])])
    for t in range(6):
        lg = pool.advance({sa: a[9 + t], sb: b[6 + t]})
        assert U.rel_err(lg[sa][None], wa[9 + t][None]) < TOL and U.rel_err(lg[sb][None], wb[6 + t][None]) < TOL
    pool.release(sb)
    for t in range(15, 40):
        assert U.rel_err(pool.advance({sa: a[t]})[sa][None], wa[t][None]) < TOL


def greedy(ref, ids, n):
    ids = list(ids)
    for _ in range(n):
        ids.append(int(ref(ids)[-1].argmax()))
    return ids[-n:]


def test_greedy_generation_through_generator_and_pool():
    from evo_amd.generation import Generator
    cfg, m, ref = cpu_model("plain")
    pool = pool_of(m, n_slots=2, top_k=1)
    prompts = ["ACGTAC", "GG", "TTTACGATCGATTA"]
    pool.generate(prompts, n_tokens=7, n_sample_per_prompt=2)
    for j, row in enumerate(pool.last_ids.tolist()):
        assert row == greedy(ref, prompts[j // 2].encode(), 7)
    g = Generator(m, pool.tok, top_k=1)
    out, _, _ = g.generate(device="cpu", input_string=prompts[0], num_tokens=7, print_generation=False)
    assert out[0].tolist() == greedy(ref, prompts[0].encode(), 7)
    out, _, _ = g.generate(device="cpu", input_string=prompts[2], num_tokens=5, print_generation=False, force_prompt_threshold=4)
    assert out[0].tolist() == greedy(ref, prompts[2].encode(), 5)


def test_scoring_entry_point():
    from evo_amd.scoring import score_sequences
    from evo_amd.tokenizer import CharLevelTokenizer
    cfg, m, ref = cpu_model("plain")
    got = score_sequences(["ACGTTA", "GGC"], m, CharLevelTokenizer(cfg["vocab"]), device="cpu")
    for s, g in zip(["ACGTTA", "GGC"], got):
        ids = [0] + list(s.encode())
        want = torch.log_softmax(ref(ids)[:-1], -1).gather(1, torch.tensor(ids[1:])[:, None]).mean()
        assert abs(g - float(want)) < 1e-4


# ------------------------------------------------------------------------------------------------ trace replay
def test_trace_replay(tmp_path, monkeypatch, capsys):
    from evo_amd import trace
    cfg, m, ref = cpu_model("order")
    a, b = U.tokens(cfg, 10, 1), U.tokens(cfg, 7, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:8], "want": [0, 7]}, {"id": "b", "tokens": b[:5], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[5:6], "want": []}, {"id": "a", "tokens": a[8:9], "want": [0]}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": b[6:7], "want": [0]}, {"id": "a", "tokens": a[9:10], "want": []}], "end": ["a", "b"]},
             {"step": 3, "entries": [{"id": "a", "tokens": b[:3], "want": [1]}], "end": ["a"]}]
    monkeypatch.setattr(trace, "load_model_dir", lambda *args, **kw: m)
    monkeypatch.setattr(sys, "stdin", io.StringIO("\n".join(json.dumps(s) for s in steps) + "\n"))
    assert trace.main(["--model", "x", "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "17"]) == 0
    assert capsys.readouterr().out.split("\n")[:4] == [f"done {i}" for i in range(4)]
    wa, wb = ref(a), ref(b)
    for n, want in ((0, wa[[0, 7]]), (1, wa[8:9]), (2, wb[6:7]), (3, wb[1:2])):
        got = np.fromfile(tmp_path / f"{n}.f32", dtype="<f4").reshape(-1, cfg["vocab"])
        assert got.shape == tuple(want.shape) and U.rel_err(got, want) < TOL
