"""GPU: whole models of the config.json families through the framework's entry points, against the plain fp64 references run one sequence at a
time.  A case is "family/configuration"."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch
from safetensors.torch import save_file

import batodra_util
import vozalorn_util
import vozalorn_util as U

FAMILIES = {"vozalorn": vozalorn_util, "batodra": batodra_util}
ALL = [f"{f}/{n}" for f, u in FAMILIES.items() for n in sorted(u.CONFIGS)]
EACH = pytest.mark.parametrize("family", sorted(FAMILIES))
pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = pytest.mark.parametrize("dt", [torch.float32, torch.bfloat16], ids=["f32", "bf16"])


NOISE = {}


def parts(name):
    u = FAMILIES[name.split("/")[0]]
    cfg = u.CONFIGS[name.split("/")[1]]
    return u, cfg, u.weights(cfg)


def tol(name, dt):
    """fp32: rounding of fp32 sums; bf16: three times the worst row that rounding alone gives (U.rounding_noise)"""
    if dt == torch.float32:
        return 2e-4
    if name not in NOISE:
        u, cfg, w = parts(name)
        ids = U.tokens(cfg, 200)
        NOISE[name] = U.rounding_noise(cfg, w, ids, u.reference(cfg, w)(ids))
    return 3 * NOISE[name][0]


@pytest.fixture(scope="module")
def cases():
    built = {}

    def get(name, dt):
        if (name, dt) not in built:
            u, cfg, w = parts(name)
            built[name, dt] = (cfg, U.build(cfg, w, dtype=dt, device=DEV), u.reference(cfg, w))
        return built[name, dt]
    return get


def pool_of(m, n_slots, **kw):
    from evo_amd.pool import DecodePool
    from evo_amd.tokenizer import CharLevelTokenizer
    return DecodePool(m, CharLevelTokenizer(m.vocab_size), n_slots=n_slots, **kw)


@DTYPES
@pytest.mark.parametrize("name", ALL)
def test_prompt_then_long_decoding(cases, name, dt):
    """A prompt in one pass, then 110 tokens one by one (every window of the configurations passes over decoded tokens); with the
    captured step where the dense shapes allow it."""
    cfg, m, ref = cases(name, dt)
    P, N = 90, 110
    ids = U.tokens(cfg, P + N)
    want = ref(ids)
    assert U.rel_err(m(torch.tensor([ids]).to(DEV))[0][0], want) < tol(name, dt)
    ipd = m.initialize_inference_params()
    m.decode_graph_replays = 0
    got = [m(torch.tensor([ids[:P]]).to(DEV), ipd)[0][0]]
    for t in range(P, P + N):
        ipd["mha"].seqlen_offset = ipd["hyena"].seqlen_offset = t
        got.append(m(torch.tensor([ids[t:t + 1]]).to(DEV), ipd)[0][0])
    m.release_decode_graph()
    err = U.row_err(torch.cat(got), want)
    assert float(err.max()) < tol(name, dt)
    if dt == torch.bfloat16:                                      # on average no worse than one rounding per op
        assert float(err.mean()) < 1.5 * NOISE[name][1]
    assert m.decode_graph and (m.decode_graph_replays == N - 1) == m._graph_shapes_ok(1)
    if dt == torch.bfloat16 and not name.endswith("/odd"):
        assert m._graph_shapes_ok(1)


@DTYPES
@pytest.mark.parametrize("cuts", [[2] * 40, [64, 16], [1, 79], [79, 1], [33, 2, 45]])
@EACH
def test_portions(cases, family, cuts, dt):
    for name in (family + "/order", family + "/window_64"):
        cfg, m, ref = cases(name, dt)
        ids = U.tokens(cfg, 80)
        ipd = m.initialize_inference_params()
        got, at = [], 0
        for n in cuts:
            ipd["mha"].seqlen_offset = ipd["hyena"].seqlen_offset = at
            got.append(m(torch.tensor([ids[at:at + n]]).to(DEV), ipd)[0][0])
            at += n
        m.release_decode_graph()
        assert U.rel_err(torch.cat(got), ref(ids)) < tol(name, dt)


@DTYPES
@pytest.mark.parametrize("name", ["vozalorn/plain", "vozalorn/odd", "vozalorn/wide_heads", "vozalorn/window_64", "batodra/plain", "batodra/odd", "batodra/grouped",
                                  "batodra/order", "batodra/window_64"])
def test_unequal_requests_and_reused_slots(cases, name, dt):
    """Waves of unequal requests share a pool: packed prompts, pooled steps (captured), early ends, slots used again."""
    cfg, m, ref = cases(name, dt)
    pool = pool_of(m, 2)
    for wave, lens in enumerate([[1, 70, 33], [130], [2, 5, 90, 64]]):
        reqs = [U.tokens(cfg, n + 14, seed=10 * wave + i) for i, n in enumerate(lens)]
        wants = [ref(r) for r in reqs]
        slots, got = pool.admit([torch.tensor(r[:n]) for r, n in zip(reqs, lens)], [list(range(n)) for n in lens], reserve=20)
        for g, w, n in zip(got, wants, lens):
            assert U.rel_err(g, w[:n]) < tol(name, dt)
        live = dict(enumerate(slots))
        for t in range(14):
            lg = pool.advance({s: reqs[i][lens[i] + t] for i, s in live.items()})
            for i, s in live.items():
                assert U.rel_err(lg[s][None], wants[i][lens[i] + t][None]) < tol(name, dt), (wave, i, t)
            if t in (3, 9) and len(live) > 1:
                pool.release(live.pop(min(live)))
        for s in live.values():
            pool.release(s)


@EACH
def test_batch_does_not_change_a_request(cases, family):
    """bf16: a prompt's logits alone and between others agree to rounding of the dense layers' different tilings."""
    cfg, m, _ = cases(family + "/window_64", torch.bfloat16)
    a, others = U.tokens(cfg, 100, 1), [U.tokens(cfg, n, n) for n in (17, 400, 64)]
    with torch.inference_mode():
        alone = m.prefill_rows([torch.tensor(a).to(DEV)], [list(range(100))])[0][0]
        mixed = m.prefill_rows([torch.tensor(t).to(DEV) for t in [others[0], a, *others[1:]]], [[], list(range(100)), [], []])[1][0]
    assert U.rel_err(mixed.float(), alone.float()) < 1.5e-2


@EACH
def test_long_prompt_in_segments(cases, family):
    """Longer than a segment of the recurrences and than many window tiles; the last tokens against the reference."""
    cfg, m, ref = cases(family + "/window_64", torch.bfloat16)
    ids = U.tokens(cfg, 1500)
    assert U.rel_err(m(torch.tensor([ids]).to(DEV))[0][0, -200:], ref(ids)[-200:]) < tol(family + "/window_64", torch.bfloat16)


def greedy(ref, ids, n):
    ids = list(ids)
    for _ in range(n):
        ids.append(int(ref(ids)[-1].argmax()))
    return ids[-n:]


@EACH
def test_greedy_generation(cases, family):
    from evo_amd.generation import generate
    cfg, m, ref = cases(family + "/plain", torch.float32)
    pool = pool_of(m, 2, top_k=1)
    prompts = ["ACGTAC", "GG", "TTTACGATCGATTA"]
    pool.generate(prompts, n_tokens=12, n_sample_per_prompt=2)
    for j, row in enumerate(pool.last_ids.tolist()):
        assert row == greedy(ref, prompts[j // 2].encode(), 12)
    out, _ = generate([prompts[0]] * 2, m, pool.tok, n_tokens=12, top_k=1, cached_generation=True, verbose=0, device=DEV)
    want = pool.tok.detokenize(greedy(ref, prompts[0].encode(), 12))
    assert out == [want, want]


@EACH
def test_bf16_generation_and_scoring_run(cases, family):
    from evo_amd.scoring import score_sequences
    cfg, m, ref = cases(family + "/window_64", torch.bfloat16)
    pool = pool_of(m, 3, top_k=1)
    pool.generate(["ACGTACGATTTA", "GG"], n_tokens=20)
    for row, lg, p in zip(pool.last_ids, pool.last_logits, ("ACGTACGATTTA", "GG")):
        want = ref(list(p.encode()) + row.tolist())[len(p) - 1:-1]
        assert U.rel_err(lg, want) < tol(family + "/window_64", torch.bfloat16)
    got = score_sequences(["ACGTTA", "GGC"], m, pool.tok, device=DEV)
    for s, g in zip(["ACGTTA", "GGC"], got):
        ids = [0] + list(s.encode())
        want = float(torch.log_softmax(ref(ids)[:-1], -1).gather(1, torch.tensor(ids[1:])[:, None]).mean())
        assert abs(g - want) < 2e-2 * abs(want)


@EACH
def test_bad_ids_raise(cases, family):
    cfg, m, _ = cases(family + "/plain", torch.bfloat16)
    with pytest.raises(IndexError):
        m(torch.tensor([[1, cfg["vocab"]]]).to(DEV))


@DTYPES
@pytest.mark.parametrize("keep,window", [(0, 6), (3, 64), (70, 40), (65, 130)])
def test_a_key_that_stands_out_at_every_distance(keep, window, dt):
    """One token that takes most of the attention: inside and outside of the window, among the kept first tokens and just behind them, in
    prompts and for decoded tokens."""
    u = batodra_util
    cfg = u.config([u.windowed(window=window, keep=keep, dim=32, rot=32, vdim=32)])
    w = u.spiky(cfg, u.weights(cfg))
    m, ref = U.build(cfg, w, dtype=dt, device=DEV), u.reference(cfg, w)
    P, T = 2 * (keep + window) // 2 + 40, 2 * (keep + window) // 2 + 90
    base = [t if t != 7 else 8 for t in U.tokens(cfg, T)]
    noise = None
    for at in sorted({0, 1, max(keep - 1, 0), keep, keep + 1, P - window, P - window + 1, P - 1, P - window + 20, T - window - 5}):
        ids = base[:at] + [7] + base[at + 1:]
        want = ref(ids)
        if dt == torch.bfloat16 and noise is None:
            noise = U.rounding_noise(cfg, w, ids, want)[0]
        limit = 2e-4 if dt == torch.float32 else 3 * noise
        assert U.rel_err(m(torch.tensor([ids]).to(DEV))[0][0], want) < limit
        ipd = m.initialize_inference_params()
        got = [m(torch.tensor([ids[:P]]).to(DEV), ipd)[0][0]]
        for t in range(P, T):
            ipd["mha"].seqlen_offset = ipd["hyena"].seqlen_offset = t
            got.append(m(torch.tensor([ids[t:t + 1]]).to(DEV), ipd)[0][0])
        m.release_decode_graph()
        assert U.rel_err(torch.cat(got), want) < limit, at


def test_caches_grow_under_the_captured_step(cases):
    """Decoding beyond the room the prompt's caches were given: they are enlarged between replays, the step is captured again."""
    cfg, m, ref = cases("batodra/window_64", torch.bfloat16)
    ids = U.tokens(cfg, 120)
    want = ref(ids)
    spare, m.spare_positions = m.spare_positions, 8
    try:
        ipd = m.initialize_inference_params()
        got = [m(torch.tensor([ids[:20]]).to(DEV), ipd)[0][0]]
        for t in range(20, 120):
            ipd["mha"].seqlen_offset = ipd["hyena"].seqlen_offset = t
            got.append(m(torch.tensor([ids[t:t + 1]]).to(DEV), ipd)[0][0])
    finally:
        m.spare_positions = spare
        m.release_decode_graph()
    assert U.rel_err(torch.cat(got), want) < tol("batodra/window_64", torch.bfloat16)


@EACH
def test_command_line(tmp_path, family):
    """scripts/generate.py on a model folder, and a trace replayed by bin/trace_run."""
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    u, cfg, w = parts(family + "/plain")
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file(w, str(tmp_path / "model.safetensors"))
    out = subprocess.run([sys.executable, "-m", "scripts.generate", "--model-dir", str(tmp_path), "--dtype", "float32", "--prompt", "ACGT",
                          "--n-samples", "1", "--n-tokens", "6", "--top-k", "1", "--verbose", "0"], cwd=root, capture_output=True, text=True, timeout=120)
    ref = u.reference(cfg, w)
    from evo_amd.tokenizer import CharLevelTokenizer
    assert out.returncode == 0, out.stderr[-2000:]
    assert CharLevelTokenizer(cfg["vocab"]).detokenize(greedy(ref, b"ACGT", 6)) in out.stdout
    ids = U.tokens(cfg, 30)
    lines = [json.dumps({"step": 0, "entries": [{"id": "r", "tokens": ids[:20], "want": [3, 19]}], "end": []})]
    lines += [json.dumps({"step": t - 19, "entries": [{"id": "r", "tokens": [ids[t]], "want": [0]}], "end": ["r"] if t == 29 else []})
              for t in range(20, 30)]
    run = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", "bfloat16", "--out", str(tmp_path),
                          "--max-tokens", "30"], input="\n".join(lines) + "\n", capture_output=True, text=True, timeout=120)
    assert run.returncode == 0, run.stderr[-2000:]
    assert [l for l in run.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(11)]
    want = ref(ids)
    got = [np.fromfile(tmp_path / f"{i}.f32", dtype="<f4").reshape(-1, cfg["vocab"]) for i in range(11)]
    assert U.rel_err(np.concatenate(got), want[[3] + list(range(19, 30))]) < tol(family + "/plain", torch.bfloat16)
