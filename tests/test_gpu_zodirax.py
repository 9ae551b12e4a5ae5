"""Zodirax on the GPU against the plain restatement in oracle/zodirax_ref.py (float64): whole prompts, decoding, portions, batches of unequal
sequences, slots that are used again, generation through the Engine; both storage types."""
import functools
import json

import pytest
import torch

from nanochat_amd.engine import Engine
from nanochat_amd.registry import load_model
from nanochat_amd.synthetic import SyntheticTokenizer
from nanochat_amd.zodirax import Zodirax
from oracle import zodirax_ref as ref
from stack_helpers import BAR, DEV, DTYPES, build_model, check, ids, judge, rel_rms, run, say, tokens, trace_runner, write_model
from zodirax_cases import CASES, config, dense, mamba, pair, scaling, weights

pytestmark = pytest.mark.gpu


@functools.lru_cache(maxsize=None)
def case_weights(name):
    return weights(CASES[name], seed=len(name))


@functools.lru_cache(maxsize=None)
def oracle_logits(name, n):
    return oracle(CASES[name], case_weights(name), tokens(CASES[name], n))


@functools.lru_cache(maxsize=None)
def case_model(name, dtype):
    return build_model(Zodirax, CASES[name], case_weights(name), dtype)


def oracle(cfg, w, toks, taps=None):
    return ref.forward(cfg, {k: v.double() for k, v in w.items()}, toks, taps)


# ------------------------------------------------------------------------------------------------ whole prompts
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(CASES))
def test_whole_prompt(name, dtype):
    say(f"whole prompt, {name}, {dtype}")
    for n in (1, 2, 45, 150, 230):
        check(run(case_model(name, dtype), tokens(CASES[name], n), [n]), oracle_logits(name, n), dtype, f"{name}, {n} tokens")


@pytest.mark.parametrize("dtype", DTYPES)
def test_residual_stream_after_every_layer(dtype):
    say(f"layer by layer, {dtype}")
    cfg, taps = CASES["odd"], []
    toks = tokens(cfg, 70)
    want = oracle(cfg, case_weights("odd"), toks, taps)
    logits, got = case_model("odd", dtype).forward_tapped(ids(toks))
    check(logits[0], want, dtype, "logits")
    assert got.shape == (len(cfg["layers"]), 1, 70, cfg["width"]) and len(taps) == len(cfg["layers"])
    for i, t in enumerate(taps):
        check(got[i, 0], t, dtype, f"layer {i}")


def mechanism(layer, mlp=None, **kw):
    return config([(layer, mlp)], width=64, vocab=50, **kw)


OFF = dict(right_heads=1, right_dim=16, right_vdim=16, right_scale=0.05)       # next to no lightning attention
MECHANISMS = {
    "window": mechanism(pair(left_scale=1.0, **OFF)),
    "window, longer than the prompt": mechanism(pair(window=500, keep_first=0, left_scale=1.0, **OFF)),
    "window of one and many first tokens": mechanism(pair(window=1, keep_first=77, left_scale=1.0, **OFF)),
    "window, peaked scores": mechanism(pair(heads=2, kv_heads=2, dim=32, vdim=32, rot_dims=32, scale=0.7, left_scale=1.0, **OFF)),
    "window, nothing turns": mechanism(pair(rot_dims=0, stretch=None, left_scale=1.0, **OFF)),
    "window, step in the stretching": mechanism(pair(stretch=scaling(factor=3.0, low=2.0, high=2.0), left_scale=1.0, **OFF)),
    "lightning": mechanism(pair(left_scale=0.05, right_scale=1.0)),
    "lightning, slow decay": mechanism(pair(left_scale=0.05, right_scale=1.0, right_heads=2, right_dim=64, right_vdim=64, decay=[0.9993, 0.9985])),
    "lightning, nothing kept and all kept": mechanism(pair(left_scale=0.05, right_scale=1.0, right_heads=2, right_dim=64, right_vdim=64, decay=[0.0, 1.0])),
    "negative scale": mechanism(pair(left_scale=-0.5, right_scale=2.0)),
    "mamba": mechanism(mamba()),
    "mamba, four taps": mechanism(mamba(inner=64, state=16, dt_rank=64, conv=4)),
    "mamba, more taps than a portion": mechanism(mamba(conv=9)),
    "mamba, states in sixteen lanes": mechanism(mamba(state=250)),
    "mamba, states in three parts of four": mechanism(mamba(state=12)),
    "swiglu": mechanism(mamba(inner=16, state=2), dense()),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MECHANISMS))
def test_each_mechanism(name, dtype):
    """One layer of each kind: prompt at once, token by token, and in portions."""
    say(f"mechanism {name}, {dtype}")
    cfg = MECHANISMS[name]
    w = weights(cfg, seed=3)
    toks = tokens(cfg, 130)
    want = oracle(cfg, w, toks)
    model = build_model(Zodirax, cfg, w, dtype)
    # (a score of tens of units turns the rounding of a bf16 query into a change of weight)
    bar = {"window, peaked scores": 0.15}.get(name) if dtype == torch.bfloat16 else None
    for cuts in ([130], [1] * 130, [2] * 65, [97, 2, 31]):
        check(run(model, toks, cuts), want, dtype, f"{name}, cuts {cuts[:3]}", bar)


def planted_mistakes():
    """(name, mechanism, function of the oracle that is replaced, replacement)."""
    def lightning_with(h, w, c, eps, act_v=None, decay=None, norm_heads=False):
        silu = ref.silu
        T, H, dk, dv = h.shape[0], c["heads"], c["dim"], c["vdim"]
        q, k, v = silu(h @ w["q"].T).view(T, H, dk), silu(h @ w["k"].T).view(T, H, dk), (act_v or silu)(h @ w["v"].T).view(T, H, dv)
        d = torch.tensor(decay or c["decay"], dtype=h.dtype)[:, None, None]
        S, o = torch.zeros(H, dk, dv, dtype=h.dtype), []
        for t in range(T):
            S = d * S + k[t][:, :, None] * v[t][:, None, :]
            o.append((S * q[t][:, :, None]).sum(1))
        o = torch.stack(o)
        o = (ref.rms_norm(o, eps, 1.0).reshape(T, -1) * w["norm"]) if norm_heads else ref.rms_norm(o.reshape(T, -1), eps, w["norm"])
        return (o * torch.sigmoid(h @ w["g"].T)) @ w["o"].T, S

    def window_with(h, w, c, eps, pos0=0, **changes):
        return WINDOW(h, dict(w, **changes.pop("weights", {})), dict(c, **changes), eps, pos0)

    def mask_with(**changes):
        return lambda i, j, m: VISIBLE(i, j, dict(m, **{k: m[k] + d for k, d in changes.items()}))

    return [("window one longer", "window", "visible", mask_with(size=1)),
            ("window one shorter", "window", "visible", mask_with(size=-1)),
            ("one first token more", "window of one and many first tokens", "visible", mask_with(keep_first=1)),
            ("one first token less", "window of one and many first tokens", "visible", mask_with(keep_first=-1)),
            ("no sink", "window", "window_attention", lambda h, w, c, eps, pos0=0: window_with(h, w, c, eps, weights={"sink": w["sink"] - 100})),
            ("no biases", "window", "window_attention",
             lambda h, w, c, eps, pos0=0: window_with(h, w, c, eps, weights={f"{n}.b": 0 * w[f"{n}.b"] for n in "qkv"})),
            ("norm per head", "window", "rms_norm", lambda x, eps, wt: RMS_NORM(x.view(-1, 2, x.shape[1] // 2), eps, 1.0).reshape(x.shape) * wt if x.shape[1] == 80
             else RMS_NORM(x, eps, wt)),
            ("frequencies not stretched", "window", "frequencies", lambda rot: FREQUENCIES({k: v for k, v in rot.items() if k != "scaling"})),
            ("no ramp in the stretching", "window", "frequencies", lambda rot: FREQUENCIES(dict(rot, scaling=dict(rot["scaling"], low=rot["scaling"]["high"])))),
            ("positions in a portion start again", "window", "rotate", lambda x, pos, rot: ROTATE(x, pos % 100, rot)),
            ("decay off by a thousandth", "lightning, slow decay", "lightning",
             lambda h, w, c, eps, state=None: lightning_with(h, w, c, eps, decay=[d * (1 - 1e-3) for d in c["decay"]])),
            ("v without silu", "lightning", "lightning", lambda h, w, c, eps, state=None: lightning_with(h, w, c, eps, act_v=lambda z: z)),
            ("heads normed one by one", "lightning", "lightning", lambda h, w, c, eps, state=None: lightning_with(h, w, c, eps, norm_heads=True)),
            ("no skip", "mamba", "selective_scan", lambda x, dt, A, B, C, D, state=None: SCAN(x, dt, A, B, C, 0 * D, state)),
            ("taps in the wrong order", "mamba", "causal_conv", lambda x, wt, b: CONV(x, wt.flip(1), b)),
            ("step sizes without softplus", "mamba", "softplus", lambda z: torch.exp(z)),
            ("norm weights not around zero", "swiglu", "layer_norm", lambda x, s, eps: RMS_NORM(x, eps, s)),
            ("gate and up exchanged", "swiglu", "dense_ff", lambda h, w: (ref.silu(h @ w["up"].T) * (h @ w["gate"].T)) @ w["down"].T)]


WINDOW, VISIBLE, SCAN, CONV, RMS_NORM, FREQUENCIES, ROTATE = (ref.window_attention, ref.visible, ref.selective_scan, ref.causal_conv, ref.rms_norm, ref.frequencies, ref.rotate)


@pytest.mark.parametrize("mistake", planted_mistakes(), ids=lambda m: m[0])
def test_bars_would_show_a_mistake(mistake, monkeypatch):
    """The same comparison with a mistake planted in the oracle fails clearly."""
    name, case, function, wrong = mistake
    say(f"planted mistake: {name}")
    cfg = MECHANISMS[case]
    w = weights(cfg, seed=3)
    toks = tokens(cfg, 120)
    good = oracle(cfg, w, toks)
    monkeypatch.setattr(ref, function, wrong)
    bad = oracle(cfg, w, toks)
    got = run(build_model(Zodirax, cfg, w, torch.float32), toks, [len(toks)])
    check(got, good, torch.float32, name)
    err = rel_rms(got, bad)[-1].item()
    print(f"{name}: {err:.2e} at the last position")
    assert err > 5 * BAR[torch.float32]


# ------------------------------------------------------------------------------------------------ a key that stands out
def standing_out(window, keep_first):
    """A model in which token 0 asks for token 1: their embeddings are opposite, and a query is minus the key of its own token, in the
    dimensions that do not turn.  The answer to a token 0 is the value of the token 1 it sees, if it sees one."""
    cfg = mechanism(pair(heads=4, kv_heads=2, dim=64, vdim=32, rot_dims=16, base=2e5, stretch=None, scale=0.25, window=window, keep_first=keep_first, left_scale=1.0,
                         **OFF))
    w = weights(cfg, seed=5)
    W, p = cfg["width"], "l0.mix.left."
    probe = torch.randn(W, generator=torch.Generator().manual_seed(9))
    w["embed"][1], w["embed"][0] = (2 * probe).bfloat16(), (-2 * probe).bfloat16()
    k = w[p + "k"].float().view(2, 64, W)
    w[p + "q"] = (-k).repeat_interleave(2, 0).reshape(-1, W).bfloat16()
    for name in ("q.b", "k.b"):
        w[p + name] = 0 * w[p + name]
    for name in ("q.norm", "k.norm"):
        w[p + name] = torch.ones_like(w[p + name])
    w["l0.norm1"] = w["l0.norm1"] + 3          # the layer's part of the stream is the larger one
    return cfg, w


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window, keep_first", [(20, 3), (64, 1), (200, 33)])
def test_keys_at_every_border(window, keep_first, dtype):
    """Every place where a window, the first tokens, a block of keys, a portion or a share of the keys begins or ends, in prompts, in portions
    and in decoding: a key just inside is the answer, the same key one place further away is not seen."""
    say(f"keys that stand out, window {window}, first {keep_first}, {dtype}")
    cfg, w = standing_out(window, keep_first)
    n = 340
    model = build_model(Zodirax, cfg, w, dtype)
    filler = torch.randint(2, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(2)).tolist()
    bar = 6e-2 if dtype == torch.bfloat16 else None
    inside = outside = 0
    for key in sorted({0, keep_first - 1, keep_first, 31, 32, 63, 64, 127, 128, 255, 256} | {n - 1 - window, n - window, n - window + 1}):
        toks = list(filler)
        toks[key] = 1
        # queries just inside and outside the window of the key, and at the end
        for at in {key + 1, key + window - 1, key + window, n - 2, n - 1}:
            if key < at < n:
                toks[at] = 0
        want = oracle(cfg, w, toks)
        without = list(toks)
        without[key] = filler[key]
        there = rel_rms(oracle(cfg, w, without), want)
        for at in (key + window - 1, key + window, n - 1):
            if key < at < n and toks[at] == 0:
                seen = at - key < window or key < keep_first
                inside, outside = inside + seen, outside + (not seen)
                # (a key out of sight moves later positions a little through the other mixer)
                assert (there[at].item() > 0.3) == seen, (key, at, there[at].item())
        check(run(model, toks, [n]), want, dtype, f"key {key}, whole", bar)
        check(run(model, toks, [63, 65, 2, 126, 64] + [1] * (n - 320)), want, dtype, f"key {key}, portions", bar)
        if key in (keep_first - 1, keep_first, 64):
            check(run(model, toks, [2] * 60 + [1] * (n - 120)), want, dtype, f"key {key}, decoding", bar)
    assert inside > 5 and outside > 3


# ------------------------------------------------------------------------------------------------ cuts
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(CASES))
def test_portions_and_decoding(name, dtype):
    say(f"cuts of one sequence, {name}, {dtype}")
    n = 150
    toks, model, want = tokens(CASES[name], n), case_model(name, dtype), oracle_logits(name, n)
    for cuts in ([2] * 75, [1] * 150, [33, 2, 64, 3, 31, 17], [149, 1], [1, 149], [64, 64, 22], [32, 32, 32, 54], [5, 140, 2, 2, 1], [96, 54], [2, 97, 51]):
        check(run(model, toks, cuts), want, dtype, f"{name}, cuts {cuts[:6]}")


def test_long_decoding():
    say("long decoding")
    for name, n in (("odd", 420), ("wide", 300)):
        toks, want = tokens(CASES[name], n), oracle_logits(name, n)
        for dtype in DTYPES:
            check(run(case_model(name, dtype), toks, [20] + [1] * (n - 20), seq_len=1000), want, dtype, f"{name}, 20 + {n - 20} tokens")


def test_results_do_not_depend_on_the_cache_length():
    say("cache length")
    toks, model = tokens(CASES["wide"], 40), case_model("wide", torch.bfloat16)
    a, b = (run(model, toks, [30] + [1] * 10, seq_len=s) for s in (40, 3000))
    assert rel_rms(a, b.double().cpu()).max().item() < 1e-2


# ------------------------------------------------------------------------------------------------ batches, slots
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["odd", "wide", "ones"])
def test_unequal_sequences_in_one_batch(name, dtype):
    """Sequences of different lengths share a cache: their decode steps equal those of each alone; then some rows end, and their
    slots take new sequences."""
    say(f"unequal batch, {name}, {dtype}")
    cfg, model, w = CASES[name], case_model(name, dtype), case_weights(name)
    lengths, steps = [3, 70, 34, 1, 129, 8], 6
    bar = 0.12 if dtype == torch.bfloat16 else None          # (the first tokens of a sequence, where a sum has few terms, round the worst)
    seqs = [tokens(cfg, n + 2 * steps, seed=10 + n) for n in lengths]
    cache = model.new_cache(len(seqs), 160)
    want = [oracle(cfg, w, s) for s in seqs]

    def admit(row, toks):
        alone = model.new_cache(1, 160)
        got = model.forward_last(ids(toks), kv_cache=alone)
        cache.load_row(row, alone)
        return got[0]

    for r, (s, n) in enumerate(zip(seqs, lengths)):
        check(admit(r, s[:n])[None], want[r][n - 1:n], dtype, f"row {r} prompt", bar)
    at = list(lengths)

    def run_steps():
        errors = [[] for _ in seqs]
        for _ in range(steps):
            col = torch.tensor([[s[p]] for s, p in zip(seqs, at)], dtype=torch.long, device=DEV)
            got = model.forward_last(col, kv_cache=cache)
            for r in range(len(seqs)):
                errors[r].append(rel_rms(got[r][None], want[r][at[r]:at[r] + 1]))
                at[r] += 1
        for r, e in enumerate(errors):
            judge(torch.cat(e), dtype, f"row {r} up to {at[r]}", bar)

    run_steps()
    assert cache.cache_seqlens.tolist() == at
    # rows 1 and 4 end; new sequences take their slots, one of them token by token from an empty slot
    cache.reset_rows([1, 4])
    seqs[1], seqs[4] = tokens(cfg, 40, seed=77), tokens(cfg, 2 * steps, seed=78)
    want[1], want[4] = oracle(cfg, w, seqs[1]), oracle(cfg, w, seqs[4])
    admit(1, seqs[1][:30])
    at[1], at[4] = 30, 0
    run_steps()


@pytest.mark.parametrize("dtype", DTYPES)
def test_prompts_of_several_rows_at_once(dtype):
    say(f"several rows, {dtype}")
    cfg, model = CASES["wide"], case_model("wide", dtype)
    seqs = [tokens(cfg, 120, seed=s) for s in (1, 2, 3)]
    want = [oracle(cfg, case_weights("wide"), s) for s in seqs]
    for cuts in ([120], [70, 2, 48], [3] * 40):
        cache = model.new_cache(3, 120)
        at, outs = 0, []
        for n in cuts:
            outs.append(model.forward(torch.tensor([s[at:at + n] for s in seqs], device=DEV), kv_cache=cache))
            at += n
        got = torch.cat(outs, dim=1)
        for r in range(3):
            check(got[r], want[r], dtype, f"row {r} of 3, cuts {cuts[:3]}")


@pytest.mark.parametrize("rows", [17, 70])
def test_many_rows_decode_together(rows):
    """More rows than one tile of the few-rows kernels, and more than they take."""
    say(f"{rows} rows")
    cfg, model, w = CASES["odd"], case_model("odd", torch.bfloat16), case_weights("odd")
    prompt = tokens(cfg, 40)
    one = model.new_cache(1, 64)
    model.forward_last(ids(prompt), kv_cache=one)
    cache = model.new_cache(rows, 64, prefill_from=one)
    tails = [tokens(cfg, 3, seed=100 + r) for r in range(rows)]
    got = [model.forward_last(torch.tensor([[t[i]] for t in tails], device=DEV), kv_cache=cache) for i in range(3)]
    for r in (0, 1, 15, 16, rows - 1):
        want = oracle(cfg, w, prompt + tails[r])[40:]
        check(torch.stack([g[r] for g in got]), want, torch.bfloat16, f"row {r} of {rows}")


def test_a_slot_is_used_again_without_a_trace():
    say("slots used again")
    model, cfg = case_model("odd", torch.bfloat16), CASES["odd"]
    cache = model.new_cache(1, 140)
    first = model.forward(ids(tokens(cfg, 50)), kv_cache=cache).clone()
    for seed, n in ((5, 117), (6, 140)):
        cache.reset()
        model.forward(ids(tokens(cfg, n, seed=seed)), kv_cache=cache)
        cache.reset()
        assert torch.equal(model.forward(ids(tokens(cfg, 50)), kv_cache=cache), first)


def test_taking_a_step_back():
    say("rewind")
    cfg, model = CASES["odd"], case_model("odd", torch.float32)
    toks = tokens(cfg, 45)
    cache = model.new_cache(1, 64)
    model.forward(ids(toks[:30]), kv_cache=cache)
    for t in toks[30:]:
        mark = cache.mark()
        model.forward_last(ids([(t + 7) % cfg["vocab"]]), kv_cache=cache)
        cache.rewind(1, mark)
        got = model.forward_last(ids([t]), kv_cache=cache)
    check(got, oracle_logits("odd", 45)[-1:], torch.float32, "after fifteen steps taken back")


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


# ------------------------------------------------------------------------------------------------ generation
def test_greedy_generation_through_the_engine(tmp_path):
    """A folder on disk, the registry, the Engine's scheduler, the sampler: the ids are the oracle's greedy ids (32-bit)."""
    say("greedy generation")
    cfg = CASES["odd"]
    w = weights(cfg, seed=31)
    write_model(tmp_path, cfg, w)
    model, info = load_model(str(tmp_path), dtype=torch.float32)
    assert type(model) is Zodirax and info["model_config"] == cfg
    prompt, new = tokens(cfg, 37, seed=4), 24
    want = list(prompt)
    for _ in range(new):
        top = oracle(cfg, w, want)[-1].topk(2)
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
    assert card["kv_bytes_per_token"] == (2 * (128 + 128) + 72 + 64) * (2 if dtype == "bfloat16" else 4)


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_replay(dtype):
    """bin/trace_run's own replay loop on two requests, one after the other, with a cache that is handed on."""
    say(f"trace replay, {dtype}")
    mod = trace_runner()
    model, toks, want = case_model("odd", dtype), tokens(CASES["odd"], 150), oracle_logits("odd", 150)
    replay = mod.Replay(model, 150)
    for name in ("a", "b"):
        check(replay.step([{"id": name, "tokens": toks[:20], "want": [0, 19]}], []), want[[0, 19]], dtype, name)
        assert replay.step([{"id": name, "tokens": toks[20:22], "want": []}], []).numel() == 0
        check(replay.step([{"id": name, "tokens": toks[22:149], "want": [3, 126]}], []), want[[25, 148]], dtype, name)
        check(replay.step([{"id": name, "tokens": toks[149:], "want": [0]}], [name]), want[149:], dtype, name)
    assert len(replay.free) == 1 and not replay.live
