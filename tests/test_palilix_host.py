"""Palilix without a GPU: configuration, registry, weight files, packing, the cache's host logic, and the oracle's own checks."""
import ctypes
import json
import re
import struct

import pytest
import torch

from nanochat_amd import _lib, registry
from nanochat_amd.build import TARGETS, is_current
from nanochat_amd.checkpoint import read_safetensors
from nanochat_amd.engine import Engine, StackCache
from nanochat_amd.palilix import Palilix, stack_config
from nanochat_amd.stack import Experts, LatentAttention, LayerStack, Retention
from oracle import palilix_ref as ref
from palilix_cases import CASES, config, latent, moe, retention, tensor_shapes, variant, weights
from stack_helpers import rel_rms, tokens


def meta_model(cfg, dtype=torch.float32):
    with torch.device("meta"):
        return Palilix.from_config(cfg, dtype)


# ------------------------------------------------------------------------------------------------ library
def test_stack_library_exports_what_the_header_declares():
    text = open(_header()).read()
    names = sorted(set(re.findall(r"\b(nc_[a-z0-9_]+)\s*\(", re.sub(r"/\*.*?\*/", "", text, flags=re.S))))
    lib = ctypes.CDLL(_lib._load("stack")._name)
    assert sorted(_lib.STACK_EXPORTS) == names and all(hasattr(lib, n) for n in names)
    assert _lib.stack_lib().nc_stack_abi_version() == 2


def _header():
    import os
    return os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "include", "nanochat_amd_stack.h")


def test_libraries_are_built_from_these_sources():
    assert all(is_current(t) for t in TARGETS), "run python -m nanochat_amd.build"


def test_struct_layouts_match_the_header(tmp_path):
    """Sizes and a few offsets as the C compiler lays them out."""
    import subprocess
    src = tmp_path / "s.c"
    src.write_text('#include <stdio.h>\n#include "%s"\nint main(){printf("%%zu %%zu %%zu %%zu %%zu %%zu %%zu %%zu %%zu", sizeof(nc_stack_layer), sizeof(nc_stack_run),'
                   'sizeof(nc_stack_model), sizeof(nc_stack_cache), offsetof(nc_stack_layer, mix), offsetof(nc_stack_model, embed),'
                   'sizeof(nc_stack_mixer), offsetof(nc_stack_mixer, kv_norm_w), offsetof(nc_stack_mixer, skip));}' % _header())
    subprocess.run(["gcc", str(src), "-o", str(tmp_path / "s")], check=True)
    got = [int(x) for x in subprocess.run([str(tmp_path / "s")], capture_output=True, text=True, check=True).stdout.split()]
    assert got == [ctypes.sizeof(_lib.StackLayer), ctypes.sizeof(_lib.StackRun), ctypes.sizeof(_lib.StackModel), ctypes.sizeof(_lib.StackCacheDesc),
                   _lib.StackLayer.mix.offset, _lib.StackModel.embed.offset, ctypes.sizeof(_lib.StackMixer), _lib.StackMixer.kv_norm_w.offset,
                   _lib.StackMixer.skip.offset]


def test_errors_come_before_any_gpu_call():
    lib = _lib.stack_lib()
    assert lib.nc_stack_linear(0, None, 64, None, None, 16, 1, 16, 64, 0, 0.0, 0, None) == -1
    assert lib.nc_stack_cache_copy(None, None, 1, 1, 16, 16, 16, None) == -1 and b"rows" in lib.nc_last_error()


# ------------------------------------------------------------------------------------------------ configuration
@pytest.mark.parametrize("name", list(CASES))
def test_tensor_table_and_sizes(name):
    cfg = CASES[name]
    sc = stack_config(cfg)
    assert LayerStack.tensor_shapes(sc) == tensor_shapes(cfg)
    assert [(i, t if t >= 0 else None) for i, _, t in sc.runs()] == ref.layer_runs(cfg)
    assert [again for _, again, _ in sc.runs()] == [bool(t) for _, t in ref.layer_runs(cfg)]
    for layer in sc.layers:
        assert layer.mixer.out % 64 == 0 and layer.mixer.cols % 16 == 0
        if isinstance(layer.mixer, LatentAttention):
            assert layer.mixer.vdim_p >= layer.mixer.vdim and layer.mixer.rank_p % 64 == 0
        else:
            assert layer.mixer.dim_p >= layer.mixer.dim and layer.mixer.vdim_p >= layer.mixer.vdim


def test_configuration_is_read_not_assumed():
    cfg = config([(retention(), None), (latent(), moe(shared=(8, 0.25)))], loop=(1, 2, 2), eps=3e-4, softcap=None)
    sc = stack_config(cfg)
    assert sc.layers[0].ff is None and isinstance(sc.layers[0].mixer, Retention) and sc.layers[0].mixer.k_scale == 40 ** -0.5
    assert isinstance(sc.layers[1].ff, Experts) and sc.layers[1].ff.shared_limit == 0.25 and sc.layers[1].ff.limit == 0.7
    assert sc.eps == 3e-4 and sc.logit_softcap == 0.0 and sc.runs() == [(0, False, -1), (1, False, 0), (1, True, 1)]
    assert stack_config(variant("wide")).runs() == [(0, False, -1), (1, False, -1), (2, False, -1)]
    with pytest.raises(ValueError):
        stack_config(variant("odd", loop={"start": 3, "stop": 1, "times": 2})).runs()
    with pytest.raises(ValueError):
        stack_config(config([(dict(latent(), type="window"), None)]))
    with pytest.raises(ValueError):
        stack_config(config([(latent(), {"kind": "dense2", "ff": 4})]))


def test_registry(tmp_path):
    assert registry.model_class("Palilix") is Palilix
    with pytest.raises(ValueError, match="unknown architecture"):
        registry.model_class("Nothing")
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Nothing"}))
    with pytest.raises(ValueError):
        registry.load_model(str(tmp_path))


def test_weight_file_reader(tmp_path):
    tensors = {"a.b": torch.randn(3, 5).bfloat16(), "c": torch.arange(7, dtype=torch.int32), "d": torch.tensor(2.5)}
    blob, header = b"", {"__metadata__": {"format": "pt"}}
    for k, t in tensors.items():
        data = t.contiguous().view(torch.uint8).numpy().tobytes() if t.dim() else struct.pack("<f", t.item())
        header[k] = {"dtype": {torch.bfloat16: "BF16", torch.int32: "I32", torch.float32: "F32"}[t.dtype], "shape": list(t.shape),
                     "data_offsets": [len(blob), len(blob) + len(data)]}
        blob += data
    head = json.dumps(header).encode()
    path = tmp_path / "model.safetensors"
    path.write_bytes(struct.pack("<Q", len(head)) + head + blob)
    got = read_safetensors(str(tmp_path))
    assert set(got) == set(tensors) and all(torch.equal(got[k], tensors[k]) and got[k].dtype == tensors[k].dtype for k in tensors)
    path.write_bytes(struct.pack("<Q", len(head)) + head + blob[:-4])
    with pytest.raises(RuntimeError):
        read_safetensors(str(tmp_path))


def test_weights_must_fit_the_model():
    cfg = CASES["odd"]
    w = weights(cfg)
    model = meta_model(cfg).load_tensors(w, "cpu")
    assert {k: t for k, t in model.named_tensors().items()}.keys() == w.keys()
    assert all(torch.equal(t, w[k]) for k, t in model.named_tensors().items())
    assert model.held_tensors()["l0.mlp.experts.down"].shape == (7, cfg["width"], 40)
    for change in (lambda d: d.pop("head"), lambda d: d.update(more=torch.zeros(1)), lambda d: d.update(head=torch.zeros(2, 2))):
        bad = dict(w)
        change(bad)
        with pytest.raises(RuntimeError):
            meta_model(cfg).load_tensors(bad, "cpu")


def test_no_cpu_fallback():
    model = meta_model(CASES["ones"]).load_tensors(weights(CASES["ones"]), "cpu")
    with pytest.raises(RuntimeError, match="GPU only"):
        model.forward(torch.zeros(1, 3, dtype=torch.long))


def test_packed_matrices_are_the_weights_in_padded_places():
    """A padded product, cut back to the heads' own sizes, is the plain product; everything else is zero."""
    cfg = CASES["odd"]
    w = {k: v.double() for k, v in weights(cfg).items()}
    sc = stack_config(cfg)
    h = torch.randn(4, cfg["width"], dtype=torch.float64)
    lat, ret = sc.layers[0].mixer, sc.layers[1].mixer
    m = ref.sub(w, "l0.mix.")
    rows, cols, extra = lat.pack(m)
    y = h @ rows.T
    q = y[:, :lat.heads * (lat.dim_p + lat.rot_p)].view(4, lat.heads, -1)
    want = (h @ m["q"].T).view(4, lat.heads, lat.dim + lat.rot_dim)
    assert torch.allclose(q[..., :lat.dim], want[..., :lat.dim]) and torch.allclose(q[..., lat.dim_p:lat.dim_p + lat.rot_dim], want[..., lat.dim:])
    assert q[..., lat.dim:lat.dim_p].abs().max() == 0 and q[..., lat.dim_p + lat.rot_dim:].numel() * q[..., lat.dim_p + lat.rot_dim:].abs().sum() == 0
    c = torch.randn(4, lat.rank, dtype=torch.float64)
    kv = (torch.nn.functional.pad(c, (0, lat.rank_p - lat.rank)) @ extra["w_ukv"].view(-1, lat.rank_p).T).view(4, lat.heads, -1)
    assert torch.allclose(kv[..., :lat.dim], (c @ m["uk"].T).view(4, lat.heads, lat.dim))
    assert torch.allclose(kv[..., lat.dim_p:lat.dim_p + lat.vdim], (c @ m["uv"].T).view(4, lat.heads, lat.vdim))
    m = ref.sub(w, "l1.mix.")
    rows, cols, extra = ret.pack(m)
    k = (h @ rows.T)[:, ret.heads * ret.dim_p:2 * ret.heads * ret.dim_p].view(4, ret.heads, ret.dim_p)
    assert torch.allclose(k[..., :ret.dim], (h @ m["k"].T).view(4, ret.heads, ret.dim)) and k[..., ret.dim:].abs().max() == 0
    o = torch.randn(4, ret.heads, ret.vdim, dtype=torch.float64)
    assert torch.allclose(torch.nn.functional.pad(o, (0, ret.vdim_p - ret.vdim)).view(4, -1) @ cols.T, o.view(4, -1) @ m["o"].T)
    ff = sc.layers[0].ff
    held = ref.sub(w, "l0.mlp.")
    held |= {k: torch.stack([held[n] for n in names]) for k, names in ff.stacked().items()}
    router, first, last, more = ff.pack(held, 128)
    hp = torch.nn.functional.pad(h, (0, 128 - cfg["width"]))
    both = hp @ first.T
    act = ref.clamped_glu(both[:, 0::2], both[:, 1::2], ff.shared_limit)
    sh = ref.sub(w, "l0.mlp.shared.")
    assert torch.allclose((act @ last.T)[:, :cfg["width"]], ref.expert(h, sh["gate"], sh["up"], sh["down"], ff.shared_limit))


def test_cost_accounting_counts_every_run():
    cfg = CASES["ones"]
    once, twice = (meta_model(dict(cfg, loop={"start": 0, "stop": 2, "times": t})) for t in (1, 2))
    head = cfg["vocab"] * cfg["width"]
    assert 2 * (once.num_active_matmul_params() - head) == twice.num_active_matmul_params() - head
    assert twice.kv_bytes_per_token() == 2 * (64 + 32) * 4
    assert twice.kv_read_bytes(10) == 10 * twice.kv_bytes_per_token() + 2 * 2 * 3 * 64 * 64 * 4
    assert twice.estimate_prefill_flops(8) > twice.estimate_decode_flops(8) > 2 * twice.num_active_matmul_params()


# ------------------------------------------------------------------------------------------------ cache
def new_cache(rows=3, seq_len=16):
    return StackCache([8, 24], [(2, 4, 4)], torch.float32, rows, seq_len, "cpu")


def test_cache_positions_and_state_buffers():
    c = new_cache()
    assert [t.shape for t in c.rows] == [(3, 16, 8), (3, 16, 24)] and [s.shape for s in c.states[0]] == [(3, 2, 4, 4)]
    first_in, first_out = c.state_buffers()
    c.advance(5)
    assert c.get_pos() == 5 and c.cache_seqlens.tolist() == [5, 5, 5]
    assert c.state_buffers()[0] is first_out and c.state_buffers()[1] is first_in
    c.cache_seqlens += 1                       # as a forward that advances the positions itself
    c.note_advanced(1)
    assert c.get_pos() == 6 and c.state_buffers()[0] is first_in
    c.rewind(1, c.mark())
    assert c.get_pos() == 5 and c.cache_seqlens.tolist() == [5, 5, 5] and c.state_buffers()[0] is first_out
    with pytest.raises(AssertionError):
        c.rewind(1)                            # only the last forward, and only once
    c.advance(2)
    c.reset_rows([1])
    assert c.cache_seqlens.tolist() == [7, 0, 7] and c._pos_max == 7 and c._host_pos == [7, 0, 7]
    with pytest.raises(AssertionError):
        c.rewind(2)                            # a row has been given back since
    c.reset_rows([0, 2])
    assert c._pos_max == 0 and c.get_pos() == 0


def test_engine_asks_the_model_for_its_cache():
    class Model:
        config = None

        def new_cache(self, batch_size, seq_len, prefill_from=None, share_prompt_reads=False):
            return (batch_size, seq_len, prefill_from, share_prompt_reads)
    assert Engine(Model(), None)._new_cache(2, 9, prefill_from="x", share_prompt_reads=True) == (2, 9, "x", True)


# ------------------------------------------------------------------------------------------------ the oracle's own checks
def test_oracle_recurrence_is_the_quadratic_sum():
    """Retention by its closed form: o_i = sum_j decay^(i-j) (q_i . k_j) v_j."""
    cfg = CASES["odd"]
    m, eps = cfg["layers"][1]["mixer"], 1e-5
    w = {k: v.double() for k, v in ref.sub(weights(cfg), "l1.mix.").items()}
    h = torch.randn(20, cfg["width"], dtype=torch.float64, generator=torch.Generator().manual_seed(0))
    got, state = ref.retention(h, w, m, eps)
    H, dk, dv = m["heads"], m["dim"], m["vdim"]
    pos = torch.arange(20)[:, None]
    q = ref.rotate((h @ w["q"].T).view(20, H, dk), pos, m["rot"]["base"], m["rot"]["dims"])
    k = ref.rotate((h @ w["k"].T).view(20, H, dk), pos, m["rot"]["base"], m["rot"]["dims"]) / dk ** 0.5
    v = (h @ w["v"].T).view(20, H, dv)
    o = torch.zeros(20, H, dv, dtype=torch.float64)
    for head, d in enumerate(m["decay"]):
        D = torch.tensor([[d ** (i - j) if j <= i else 0.0 for j in range(20)] for i in range(20)], dtype=torch.float64)
        o[:, head] = ((q[:, head] @ k[:, head].T) * D) @ v[:, head]
    y = ref.rms_norm(o, eps).reshape(20, -1) * ref.silu(h @ w["g"].T)
    assert torch.allclose(got, y @ w["o"].T)
    again, end = ref.retention(h[:11], w, m, eps)
    rest, end = ref.retention(h[11:], w, m, eps, pos0=11, state=end)
    assert torch.allclose(torch.cat([again, rest]), got) and torch.allclose(end, state)


def test_oracle_rotation_keeps_relative_positions():
    x, y = torch.randn(2, 12, dtype=torch.float64)
    dots = [(ref.rotate(x[None], torch.tensor([p]), 100.0, 8)[0] @ ref.rotate(y[None], torch.tensor([p + 3]), 100.0, 8)[0]).item() for p in (0, 5, 4000)]
    assert max(dots) - min(dots) < 1e-9
    assert torch.equal(ref.rotate(x[None], torch.tensor([7]), 100.0, 8)[0, 8:], x[8:])


def test_oracle_routes_the_highest_scores():
    h, r = torch.randn(6, 10, dtype=torch.float64), torch.randn(9, 10, dtype=torch.float64)
    idx, wt = ref.route(h, r, 4)
    s = torch.softmax(h @ r.T, -1)
    for t in range(6):
        assert sorted(idx[t].tolist()) == sorted(s[t].argsort(descending=True)[:4].tolist())
        assert torch.allclose(wt[t], s[t][idx[t]] / s[t][idx[t]].sum()) and abs(wt[t].sum().item() - 1) < 1e-12


def test_oracle_is_causal_and_every_mechanism_matters():
    cfg = CASES["odd"]
    w = {k: v.double() for k, v in weights(cfg).items()}
    toks = tokens(cfg, 30)
    full = ref.forward(cfg, w, toks)
    assert rel_rms(ref.forward(cfg, w, toks[:21]), full[:21]).max() < 1e-12
    g = torch.Generator().manual_seed(4)
    for name in w:                              # no tensor is a passenger
        if re.search(r"e[1-9]+\.", name):       # (an expert may not be chosen in so few tokens)
            continue
        noise = torch.randn(w[name].shape, generator=g, dtype=torch.float64) * w[name].std()
        assert rel_rms(ref.forward(cfg, dict(w, **{name: w[name] + noise}), toks), full).max() > 1e-2, name
