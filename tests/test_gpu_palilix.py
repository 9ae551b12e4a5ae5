"""Palilix on the GPU against the plain restatement in oracle/palilix_ref.py (float64): whole prompts, decoding, portions, batches of
unequal sequences, slots that are used again, generation through the Engine; both storage types."""
import functools
import json

import pytest
import torch

from nanochat_amd import ops
from nanochat_amd.engine import Engine
from nanochat_amd.palilix import Palilix
from nanochat_amd.registry import load_model
from nanochat_amd.synthetic import SyntheticTokenizer
from oracle import palilix_ref as ref
from palilix_cases import CASES, config, dense, latent, moe, retention, variant, weights
from stack_helpers import BAR, DEV, DTYPES, build_model, check, ids, judge, rel_rms, run, say, tokens, trace_runner, write_model

pytestmark = pytest.mark.gpu


@functools.lru_cache(maxsize=None)
def case_weights(name):
    return weights(CASES[name], seed=len(name))


@functools.lru_cache(maxsize=None)
def oracle_logits(name, n):
    cfg = CASES[name]
    return ref.forward(cfg, {k: v.double() for k, v in case_weights(name).items()}, tokens(cfg, n))


@functools.lru_cache(maxsize=None)
def case_model(name, dtype):
    return build(CASES[name], case_weights(name), dtype)


def build(cfg, w, dtype):
    return build_model(Palilix, cfg, w, dtype)


# ------------------------------------------------------------------------------------------------ linears
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", [0, 1, 2, 3, 6, 7])
def test_linear_kernels(dtype, kind):
    say(f"linears, kind {kind}, {dtype}")
    g = torch.Generator().manual_seed(kind)
    for M, N, K in [(1, 16, 64), (3, 48, 128), (16, 1040, 192), (17, 96, 64), (33, 144, 448), (64, 80, 704), (65, 256, 64), (129, 144, 320), (300, 1072, 128)]:
        a, w = torch.randn(M, K, generator=g).to(dtype), (torch.randn(N, K, generator=g) / K ** 0.5).to(dtype)
        want = a.double() @ w.double().T
        if kind == 1:
            want = ref.gelu_tanh(want)
        elif kind == 2:
            want = ref.clamped_glu(want[:, 0::2], want[:, 1::2], 0.6)
        elif kind == 6:
            want = ref.silu(want)
        elif kind == 7:
            want = ref.silu(want[:, 0::2]) * want[:, 1::2]
        for kernel in (1, 2, 3, 4):
            got = ops.stack_linear(a.to(DEV), w.to(DEV), kind=kind, limit=0.6, kernel=kernel).cpu()
            tol = 1e-2 if got.dtype == torch.bfloat16 else 2e-5
            assert torch.allclose(got.double(), want, rtol=tol, atol=tol), (M, N, K, kernel, (got.double() - want).abs().max().item())


# ------------------------------------------------------------------------------------------------ whole prompts
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(CASES))
def test_whole_prompt(name, dtype):
    say(f"whole prompt, {name}, {dtype}")
    for n in (1, 2, 45, 150):
        toks = tokens(CASES[name], n)
        check(run(case_model(name, dtype), toks, [n]), oracle_logits(name, n), dtype, f"{name}, {n} tokens")


@pytest.mark.parametrize("dtype", DTYPES)
def test_residual_stream_after_every_run(dtype):
    say(f"layer by layer, {dtype}")
    cfg, taps = CASES["odd"], []
    toks = tokens(cfg, 70)
    want = ref.forward(cfg, {k: v.double() for k, v in case_weights("odd").items()}, toks, taps)
    model = case_model("odd", dtype)
    logits, got = model.forward_tapped(ids(toks))
    check(logits[0], want, dtype, "logits")
    assert got.shape == (len(ref.layer_runs(cfg)), 1, 70, cfg["width"]) == (len(taps), 1, 70, cfg["width"])
    for i, t in enumerate(taps):
        check(got[i, 0], t, dtype, f"run {i}")


def mechanism(layer, mlp=None, **kw):
    return config([(layer, mlp)], width=64, vocab=50, **kw)


MECHANISMS = {
    "latent": mechanism(latent()),
    "latent, peaked scores": mechanism(latent(heads=2, dim=32, rot_dim=32, vdim=32, kv_rank=64, scale=1.5)),
    "retention": mechanism(retention()),
    "retention, slow decay": mechanism(retention(heads=2, dim=64, vdim=64, rot_dims=32, decay=[0.9993, 0.9985])),
    "retention, nothing kept and all kept": mechanism(retention(heads=2, dim=64, vdim=64, rot_dims=32, decay=[0.0, 1.0])),
    "dense": mechanism(retention(heads=1, dim=16, vdim=16, rot_dims=8), dense()),
    "experts": mechanism(retention(heads=1, dim=16, vdim=16, rot_dims=8), moe(experts=33, top=5)),
    "experts and shared": mechanism(retention(heads=1, dim=16, vdim=16, rot_dims=8), moe(shared=(40, 0.2))),
    "loop": mechanism(latent(heads=2), loop=(0, 1, 4)),
    "no layers in the loop": mechanism(latent(heads=2), loop=(1, 1, 2)),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MECHANISMS))
def test_each_mechanism(name, dtype):
    """One layer of each kind: prompt at once, and token by token."""
    say(f"mechanism {name}, {dtype}")
    cfg = MECHANISMS[name]
    w = weights(cfg, seed=3)
    toks = tokens(cfg, 100)
    want = ref.forward(cfg, {k: v.double() for k, v in w.items()}, toks)
    model = build(cfg, w, dtype)
    # (a score of tens of units turns the rounding of a bf16 query into a change of weight)
    # and a head that sees one key only answers with its value times the sign of the score
    bar = {"latent, peaked scores": 0.15, "retention, nothing kept and all kept": 0.15}.get(name) if dtype == torch.bfloat16 else None
    check(run(model, toks, [100]), want, dtype, name, bar)
    check(run(model, toks, [1] * 100), want, dtype, name + ", token by token", bar)


def planted_mistakes():
    """(name, mechanism, function of the oracle that is replaced, replacement)."""
    def half_of_it(g, u, lim):
        return g.clamp(max=lim) * torch.sigmoid(1.702 * g.clamp(max=lim)) * (u.clamp(max=lim) + 1)

    def gate_on_both_sides(g, u, lim):
        return g.clamp(-lim, lim) * torch.sigmoid(1.702 * g.clamp(-lim, lim)) * (u.clamp(-lim, lim) + 1)

    return [("decay off by a thousandth", "retention, slow decay", "retention",
             lambda h, wt, c, eps: RETENTION(h, wt, dict(c, decay=[d * (1 - 1e-3) for d in c["decay"]]), eps)),
            ("rotation base a hundredth off", "latent, peaked scores", "rotate", lambda x, pos, base, dims: ROTATE(x, pos, base * 1.01, dims)),
            ("epsilon forgotten in the latent's norm", "latent", "rms_norm", lambda x, eps, weight=None: RMS_NORM(x, 0.03, weight)),
            ("weights not divided by their sum", "experts", "route", lambda h, r, top: torch.softmax(h @ r.T, -1).topk(top, -1)[::-1]),
            ("up not clamped below", "experts and shared", "clamped_glu", half_of_it),
            ("gate clamped below", "experts and shared", "clamped_glu", gate_on_both_sides),
            ("erf-like gelu", "dense", "gelu_tanh", lambda z: torch.nn.functional.gelu(z)),
            ("embedding output not added again", "loop", "layer_runs", lambda cfg: [(i, t if t == 0 else None) for i, t in LAYER_RUNS(cfg)])]


RETENTION, LAYER_RUNS, ROTATE, RMS_NORM = ref.retention, ref.layer_runs, ref.rotate, ref.rms_norm


@pytest.mark.parametrize("mistake", planted_mistakes(), ids=lambda m: m[0])
def test_bars_would_show_a_mistake(mistake, monkeypatch):
    """The same comparison with a mistake planted in the oracle fails clearly."""
    name, case, function, wrong = mistake
    say(f"planted mistake: {name}")
    cfg = MECHANISMS[case]
    w = weights(cfg, seed=3)
    toks = tokens(cfg, 100)
    w64 = {k: v.double() for k, v in w.items()}
    good = ref.forward(cfg, w64, toks)
    monkeypatch.setattr(ref, function, wrong)
    bad = ref.forward(cfg, w64, toks)
    got = run(build(cfg, w, torch.float32), toks, [len(toks)])
    check(got, good, torch.float32, name)
    err = rel_rms(got, bad)[-1].item()
    print(f"{name}: {err:.2e} at the last position")
    assert err > 5 * BAR[torch.float32]


# ------------------------------------------------------------------------------------------------ a far key that stands out
@pytest.mark.parametrize("dtype", DTYPES)
def test_keys_at_the_borders_of_the_kernels_blocks(dtype):
    """One key stands out for one query: the query's answer is that key's value.  Every place where a block of keys, a portion or a share
    of the keys begins or ends is visited, in prompts, in portions and in decoding."""
    say(f"keys that stand out, {dtype}")
    cfg = mechanism(latent(heads=2, dim=32, rot_dim=32, vdim=32, kv_rank=64, scale=0.3, base=2e5))
    w = weights(cfg, seed=5)
    # token 0 asks for token 1: their embeddings are opposite, and a query's unrotated part is minus the unrotated key of its own token
    W = cfg["width"]
    probe = torch.randn(W, generator=torch.Generator().manual_seed(9))
    w["embed"][1], w["embed"][0] = (3 * probe).bfloat16(), (-3 * probe).bfloat16()
    uk, q = w["l0.mix.uk"].float().view(2, 32, 64), w["l0.mix.q"].float().view(2, 64, W)
    q[:, :32] = -1.5 * uk @ w["l0.mix.dkv"].float()[:64]
    w["l0.mix.q"], w["l0.mix.o"] = q.view(-1, W).bfloat16(), 4 * w["l0.mix.o"]
    w64 = {k: v.double() for k, v in w.items()}
    n = 330
    model = build(cfg, w, dtype)
    g = torch.Generator().manual_seed(2)
    filler = torch.randint(2, cfg["vocab"], (n,), generator=g).tolist()
    bar = 6e-2 if dtype == torch.bfloat16 else None
    for key in (0, 1, 31, 32, 63, 64, 127, 128, 255, 256):
        toks = list(filler)
        toks[key] = 1
        for at in (key + 1, key + 2, 319, 320, n - 1):
            toks[at] = 0
        want = ref.forward(cfg, w64, toks)
        shifted = list(toks)
        shifted[key] = filler[key]
        there = rel_rms(ref.forward(cfg, w64, shifted), want)[n - 1].item()
        assert there > 0.3, (key, there)              # the answer at the end rests on this key
        check(run(model, toks, [n]), want, dtype, f"key {key}, whole", bar)
        check(run(model, toks, [63, 65, 2, 126, 64] + [1] * (n - 320)), want, dtype, f"key {key}, portions", bar)


# ------------------------------------------------------------------------------------------------ cuts
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["odd", "wide", "ones", "large_heads"])
def test_portions_and_decoding(name, dtype):
    say(f"cuts of one sequence, {name}, {dtype}")
    n = 150
    toks, model, want = tokens(CASES[name], n), case_model(name, dtype), oracle_logits(name, n)
    for cuts in ([2] * 75, [1] * 150, [33, 2, 64, 3, 31, 17], [149, 1], [1, 149], [64, 64, 22], [32, 32, 32, 54], [5, 140, 2, 2, 1]):
        check(run(model, toks, cuts), want, dtype, f"{name}, cuts {cuts[:6]}")


def test_long_decoding():
    say("long decoding")
    name, n = "odd", 420
    toks, want = tokens(CASES[name], n), oracle_logits(name, n)
    for dtype in DTYPES:
        check(run(case_model(name, dtype), toks, [20] + [1] * (n - 20), seq_len=1000), want, dtype, "20 + 400 tokens")


def test_results_do_not_depend_on_the_cache_length():
    say("cache length")
    toks, model = tokens(CASES["wide"], 40), case_model("wide", torch.bfloat16)
    a, b = (run(model, toks, [30] + [1] * 10, seq_len=s) for s in (40, 3000))
    assert rel_rms(a, b.double().cpu()).max().item() < 1e-2


# ------------------------------------------------------------------------------------------------ batches, slots
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["odd", "wide"])
def test_unequal_sequences_in_one_batch(name, dtype):
    """Sequences of different lengths share a cache: their decode steps equal those of each alone; then some rows end, and their
    slots take new sequences."""
    say(f"unequal batch, {name}, {dtype}")
    cfg, model = CASES[name], case_model(name, dtype)
    lengths, steps = [3, 70, 34, 1, 129], 6
    seqs = [tokens(cfg, n + 2 * steps, seed=10 + n) for n in lengths]
    w64 = {k: v.double() for k, v in case_weights(name).items()}
    cache = model.new_cache(len(seqs), 160)
    want = [ref.forward(cfg, w64, s) for s in seqs]

    def admit(row, toks):
        alone = model.new_cache(1, 160)
        got = model.forward_last(ids(toks), kv_cache=alone)
        cache.load_row(row, alone)
        return got[0]

    for r, (s, n) in enumerate(zip(seqs, lengths)):
        check(admit(r, s[:n])[None], want[r][n - 1:n], dtype, f"row {r} prompt")
    at = list(lengths)

    def step_all():
        col = torch.tensor([[s[p]] for s, p in zip(seqs, at)], dtype=torch.long, device=DEV)
        got = model.forward_last(col, kv_cache=cache)
        for r in range(len(seqs)):
            errors[r].append(rel_rms(got[r][None], want[r][at[r]:at[r] + 1]))
            at[r] += 1

    def run_steps():
        for e in errors:
            e.clear()
        for _ in range(steps):
            step_all()
        for r, e in enumerate(errors):
            judge(torch.cat(e), dtype, f"row {r} up to {at[r]}")
    errors = [[] for _ in seqs]
    run_steps()
    assert cache.cache_seqlens.tolist() == at
    # rows 1 and 4 end; new sequences take their slots, one of them token by token from an empty slot
    cache.reset_rows([1, 4])
    seqs[1], seqs[4] = tokens(cfg, 40, seed=77), tokens(cfg, 2 * steps, seed=78)
    want[1], want[4] = ref.forward(cfg, w64, seqs[1]), ref.forward(cfg, w64, seqs[4])
    admit(1, seqs[1][:30])
    at[1], at[4] = 30, 0
    run_steps()


@pytest.mark.parametrize("dtype", DTYPES)
def test_prompts_of_several_rows_at_once(dtype):
    say(f"several rows, {dtype}")
    cfg, model = CASES["wide"], case_model("wide", dtype)
    w64 = {k: v.double() for k, v in case_weights("wide").items()}
    seqs = [tokens(cfg, 90, seed=s) for s in (1, 2, 3)]
    for cuts in ([90], [40, 2, 48], [3] * 30):
        cache = model.new_cache(3, 90)
        at, outs = 0, []
        for n in cuts:
            outs.append(model.forward(torch.tensor([s[at:at + n] for s in seqs], device=DEV), kv_cache=cache))
            at += n
        got = torch.cat(outs, dim=1)
        for r, s in enumerate(seqs):
            check(got[r], ref.forward(cfg, w64, s), dtype, f"row {r} of 3, cuts {cuts[:3]}")


def test_a_slot_is_used_again_without_a_trace():
    say("slots used again")
    model, cfg = case_model("odd", torch.bfloat16), CASES["odd"]
    cache = model.new_cache(1, 120)
    first = model.forward(ids(tokens(cfg, 50)), kv_cache=cache).clone()
    for seed in (5, 6):
        cache.reset()
        model.forward(ids(tokens(cfg, 117, seed=seed)), kv_cache=cache)
        cache.reset()
        assert torch.equal(model.forward(ids(tokens(cfg, 50)), kv_cache=cache), first)


def test_taking_a_step_back():
    say("rewind")
    cfg, model = CASES["odd"], case_model("odd", torch.float32)
    toks = tokens(cfg, 40)
    cache = model.new_cache(1, 64)
    model.forward(ids(toks[:30]), kv_cache=cache)
    for t in toks[30:]:
        mark = cache.mark()
        model.forward_last(ids([(t + 7) % cfg["vocab"]]), kv_cache=cache)
        cache.rewind(1, mark)
        got = model.forward_last(ids([t]), kv_cache=cache)
    check(got, oracle_logits("odd", 40)[-1:], torch.float32, "after ten steps taken back")
    with pytest.raises(AssertionError):
        cache.rewind(2)


def test_chosen_places_and_errors():
    say("forward_at, refused calls")
    cfg, model = CASES["odd"], case_model("odd", torch.float32)
    toks = tokens(cfg, 33)
    every = model.forward(ids(toks))[0]
    assert torch.equal(model.forward_at(ids(toks), [32, 0, 5]), every[[32, 0, 5]])
    cache = model.new_cache(1, 33)
    assert model.forward_at(ids(toks[:20]), [], kv_cache=cache).shape == (0, cfg["vocab"]) and cache.get_pos() == 20
    assert torch.allclose(model.forward_at(ids(toks[20:]), [12], kv_cache=cache), every[32:], rtol=0, atol=1e-4)
    with pytest.raises(AssertionError):
        model.forward(ids([1]), kv_cache=cache)                      # full
    with pytest.raises(IndexError):
        model.forward(ids([1, cfg["vocab"]]))
    with pytest.raises(ValueError):
        Palilix.from_config(cfg, torch.float16)


# ------------------------------------------------------------------------------------------------ generation
def test_greedy_generation_through_the_engine(tmp_path):
    """A folder on disk, the registry, the Engine's scheduler, the sampler: the ids are the oracle's greedy ids (32-bit)."""
    say("greedy generation")
    cfg = variant("odd", logit_scale=2.5)
    w = weights(cfg, seed=29)
    write_model(tmp_path, cfg, w)
    model, info = load_model(str(tmp_path), dtype=torch.float32)
    assert type(model) is Palilix and info["model_config"] == cfg
    w64 = {k: v.double() for k, v in w.items()}
    prompt, new = tokens(cfg, 37, seed=4), 24
    want = list(prompt)
    for _ in range(new):
        top = ref.forward(cfg, w64, want)[-1].topk(2)
        assert (top.values[0] - top.values[1]).item() > 1e-3           # no close call: the ids must agree
        want.append(top.indices[0].item())
    engine = Engine(model, SyntheticTokenizer())
    for kw in ({}, {"num_samples": 3}, {"prefill_chunk": 2}, {"prefill_chunk": 16, "num_samples": 2}):
        out, masks = engine.generate_batch(prompt, max_tokens=new, temperature=0.0, **kw)
        assert out == [want] * kw.get("num_samples", 1), kw
        assert masks[0] == [0] * len(prompt) + [1] * new
    # bf16, sampled: the stream is reproducible, rows differ
    half, _ = load_model(str(tmp_path))
    runs = [Engine(half, SyntheticTokenizer()).generate_batch(prompt, num_samples=4, max_tokens=12, temperature=1.0, top_k=20, seed=5)[0] for _ in range(2)]
    assert runs[0] == runs[1] and len({tuple(r) for r in runs[0]}) > 1


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_harness_on_a_model_folder(tmp_path, capsys, dtype):
    say(f"infer_bench --model, {dtype}")
    from nanochat_amd import infer_bench
    write_model(tmp_path, CASES["wide"], case_weights("wide"))
    infer_bench.main(["--model", str(tmp_path), "--dtype", dtype, "--prompt-tokens", "40", "--decode-tokens", "6", "--batch-sizes", "1,3"])
    card = json.loads(capsys.readouterr().out.strip().splitlines()[-1])
    assert card["model_config"] == CASES["wide"] and [s["batch_size"] for s in card["sweep"]] == [1, 3]
    assert card["kv_bytes_per_token"] == (512 + 64) * (2 if dtype == "bfloat16" else 4)


class ForcingTokenizer(SyntheticTokenizer):
    """Every sequence meets the tool-use tokens at once: <|python_start|> is whatever the model likes to say, so that the state machine
    forces tokens of its own and the step run ahead is taken back."""

    def __init__(self, start, end, out):
        self.ids = {"<|python_start|>": start, "<|python_end|>": end, "<|output_start|>": out, "<|output_end|>": out + 1, "<|assistant_end|>": 1 << 30}

    def encode_special(self, s):
        return self.ids[s]

    def encode(self, s, prepend=None):
        return [2, 3]

    def decode(self, toks):
        return "1+1"


def test_forced_tokens_take_the_step_back():
    say("forced tokens")
    cfg, model = CASES["odd"], case_model("odd", torch.float32)
    prompt = tokens(cfg, 9, seed=8)
    plain = Engine(model, SyntheticTokenizer()).generate_batch(prompt, max_tokens=10, temperature=0.0)[0][0][9:]
    # the second token opens the tool block, the first later one that differs from both its neighbours in kind closes it
    start = plain[1]
    end = next(t for i, t in enumerate(plain) if i >= 3 and t != start)
    tok = ForcingTokenizer(start, end, 120)
    out, masks = Engine(model, tok).generate_batch(prompt, max_tokens=24, temperature=0.0)
    assert 0 in masks[0][9:], "no token was forced"
    # the same ids, teacher-forced through the oracle: every sampled token is its greedy choice
    w64 = {k: v.double() for k, v in case_weights("odd").items()}
    logits = ref.forward(cfg, w64, out[0])
    for i in range(9, len(out[0])):
        if masks[0][i]:
            assert logits[i - 1].argmax().item() == out[0][i], i


def test_trace_replay(tmp_path):
    """bin/trace_run's own replay loop on two requests, one after the other, with a cache that is handed on."""
    say("trace replay")
    mod = trace_runner()
    cfg, model = CASES["odd"], case_model("odd", torch.float32)
    toks = tokens(cfg, 45)
    want = oracle_logits("odd", 45)
    replay = mod.Replay(model, 45)
    for name in ("a", "b"):
        got = replay.step([{"id": name, "tokens": toks[:20], "want": [0, 19]}], [])
        check(got, want[[0, 19]], torch.float32, name)
        assert replay.step([{"id": name, "tokens": toks[20:22], "want": []}], []).numel() == 0
        got = replay.step([{"id": name, "tokens": toks[22:44], "want": [3]}], [])
        check(got, want[25:26], torch.float32, name)
        got = replay.step([{"id": name, "tokens": toks[44:], "want": [0]}], [name])
        check(got, want[44:], torch.float32, name)
    assert len(replay.free) == 1 and not replay.live
    grown = mod.Replay(model, 10)                      # more tokens than were announced
    grown.step([{"id": "c", "tokens": toks[:10], "want": []}], [])
    check(grown.step([{"id": "c", "tokens": toks[10:45], "want": [34]}], ["c"]), want[44:], torch.float32, "grown")
