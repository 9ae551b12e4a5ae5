"""Zodirax without a GPU: configuration, registry, packing, cost accounting, cache shapes, and the oracle's own checks."""
import math

import pytest
import torch

from nanochat_amd import registry
from nanochat_amd.engine import StackCache
from nanochat_amd.stack import DenseSwiglu, LayerStack, Retention, Rotation, SelectiveScan, SideBySide, WindowAttention
from nanochat_amd.zodirax import Zodirax, stack_config
from oracle import zodirax_ref as ref
from stack_helpers import rel_rms, tokens
from zodirax_cases import CASES, config, dense, mamba, pair, scaling, tensor_shapes, weights


def meta_model(cfg, dtype=torch.float32):
    with torch.device("meta"):
        return Zodirax.from_config(cfg, dtype)


# ------------------------------------------------------------------------------------------------ configuration
@pytest.mark.parametrize("name", list(CASES))
def test_tensor_table_and_sizes(name):
    cfg = CASES[name]
    sc = stack_config(cfg)
    assert LayerStack.tensor_shapes(sc) == tensor_shapes(cfg)
    assert sc.runs() == [(i, False, -1) for i in range(len(cfg["layers"]))]
    for layer in sc.layers:
        assert sum(m.out for m in layer.mixers) % 64 == 0 and all(m.cols % 16 == 0 and m.out % 16 == 0 for m in layer.mixers)
        for m in layer.mixers:
            if isinstance(m, SelectiveScan):
                assert m.state_p >= m.state and m.state_p % 4 == 0 and m.state_shape == (m.state_p + m.conv - 1, m.inner_p)
            else:
                assert m.dim_p >= m.dim and m.vdim_p >= m.vdim


def test_configuration_is_read_not_assumed():
    cfg = config([(mamba(), None), (pair(stretch=None, left_scale=0.25, right_scale=-1.5), dense(ff=10))], eps=3e-4, scale=7.0)
    sc = stack_config(cfg)
    scan, both = sc.layers[0].mixer, sc.layers[1].mixer
    assert sc.layers[0].ff is None and (scan.inner, scan.state, scan.dt_rank, scan.conv) == (90, 5, 7, 3)
    assert isinstance(both, SideBySide) and isinstance(both.left, WindowAttention) and isinstance(both.right, Retention) and isinstance(sc.layers[1].ff, DenseSwiglu)
    assert (both.left.out_scale, both.right.out_scale) == (0.25, -1.5) and both.left.scale == 0.21 and (both.left.window, both.left.keep_first) == (11, 3)
    assert both.left.rotation == Rotation(700.0, 28) and both.right.rotation.dims == 0 and both.right.k_scale == 1.0 and both.right.silu_qkv and both.right.joint_norm
    assert sc.eps == 3e-4 and sc.embed_scale == 7.0 and sc.tied_head and sc.norm_offset == 1.0 and sc.block == "post_norm"
    rot = stack_config(config([(pair(), None)])).layers[0].mixer.left.rotation
    assert rot == Rotation(700.0, 28, factor=4.0, low=1.0, high=3.0, original=64.0)
    with pytest.raises(ValueError):
        stack_config(config([(dict(pair(), type="serial"), None)]))
    with pytest.raises(ValueError):
        stack_config(config([(mamba(), {"kind": "moe"})]))
    with pytest.raises(AssertionError):
        stack_config(config([(pair(heads=5, kv_heads=2), None)]))


@pytest.mark.parametrize("rot", [{"base": 500.0, "dims": 30}, {"base": 500.0, "dims": 30, "scaling": scaling()}, {"base": 9000.0, "dims": 64, "scaling": scaling(low=2.0, high=2.0)},
                                 {"base": 10.0, "dims": 2, "scaling": scaling(factor=1.0)}, {"base": 1e5, "dims": 128, "scaling": scaling(8.0, 0.5, 6.0, 4096)}])
def test_frequencies(rot):
    cfg = config([(pair(dim=128), None)])
    cfg["layers"][0]["mixer"]["left"]["rot"] = rot
    got = stack_config(cfg).layers[0].mixer.left.rotation.frequencies()
    assert torch.allclose(got, torch.tensor(ref.frequencies(rot), dtype=torch.float64), rtol=1e-12, atol=0)
    plain = torch.tensor([rot["base"] ** (-2.0 * i / rot["dims"]) for i in range(rot["dims"] // 2)], dtype=torch.float64)
    s = rot.get("scaling")
    if s and s["factor"] > 1 and rot["dims"] > 2:              # the fast ones stay, the slow ones are stretched
        assert got[0] == plain[0] and math.isclose(got[-1], plain[-1] / s["factor"]) and bool((got <= plain).all())


def test_registry_and_weights_must_fit():
    assert registry.model_class("Zodirax") is Zodirax
    cfg = CASES["odd"]
    w = weights(cfg)
    model = meta_model(cfg).load_tensors(w, "cpu")
    assert all(torch.equal(t, w[k]) for k, t in model.named_tensors().items()) and set(model.named_tensors()) == set(w)
    meta_model(cfg).load_tensors(dict(w, **{"l1.norm2": torch.zeros(cfg["width"])}), "cpu")      # the norm of a feed-forward that is not there
    for change in (lambda d: d.pop("l0.mix.left.sink"), lambda d: d.update(head=w["embed"]), lambda d: d.update({"l0.norm2": torch.zeros(2)})):
        bad = dict(w)
        change(bad)
        with pytest.raises(RuntimeError):
            meta_model(cfg).load_tensors(bad, "cpu")
    with pytest.raises(RuntimeError, match="GPU only"):
        model.forward(torch.zeros(1, 3, dtype=torch.long))


def test_packed_matrices_are_the_weights_in_padded_places():
    """A padded product, cut back to the heads' own sizes, is the plain product; everything else is zero."""
    cfg = CASES["odd"]
    w = {k: v.double() for k, v in weights(cfg).items()}
    sc = stack_config(cfg)
    h = torch.randn(4, cfg["width"], dtype=torch.float64)
    a, m = sc.layers[0].mixer.left, ref.sub(w, "l0.mix.left.")
    rows, cols, extra = a.pack(m)
    y = h @ rows.T + extra["qkv_bias"].double()
    assert y.shape == (4, a.cols)
    at = 0
    for name, n, d, d_p in (("q", a.heads, a.dim, a.dim_p), ("k", a.kv_heads, a.dim, a.dim_p), ("v", a.kv_heads, a.vdim, a.vdim_p)):
        got, at = y[:, at:at + n * d_p].view(4, n, d_p), at + n * d_p
        assert torch.allclose(got[..., :d], (h @ m[name].T + m[name + ".b"]).view(4, n, d)) and got[..., d:].abs().sum() == 0
    o = torch.randn(4, a.heads, a.vdim, dtype=torch.float64)
    assert torch.allclose(torch.nn.functional.pad(o, (0, a.vdim_p - a.vdim)).view(4, -1) @ cols.T, o.view(4, -1) @ m["o"].T)
    assert extra["q_norm_w"].shape == (a.heads, a.dim_p) and torch.equal(extra["q_norm_w"][:, :a.dim].reshape(-1).double(), m["q.norm"])
    s, m = sc.layers[2].mixer, ref.sub(w, "l2.mix.")
    rows, cols, extra = s.pack(m)
    x, z = (h @ rows.T).split([s.inner_p, s.inner_p], -1)
    assert torch.allclose(torch.cat([x[:, :s.inner], z[:, :s.inner]], -1), h @ m["in"].T) and x[:, s.inner:].abs().sum() == 0
    u = torch.randn(4, s.inner, dtype=torch.float64)
    p = torch.nn.functional.pad(u, (0, s.inner_p - s.inner)) @ extra["w_x"].T
    step, B, C = p.split([s.dt_rank_p, s.bc_p, s.bc_p], -1)
    assert torch.allclose(torch.cat([step[:, :s.dt_rank], B[:, :s.state], C[:, :s.state]], -1), u @ m["x"].T)
    assert torch.allclose((step @ extra["w_dt"].T)[:, :s.inner], step[:, :s.dt_rank] @ m["dt"].T) and torch.equal(extra["w_dt_t"], extra["w_dt"].T)
    assert torch.allclose(torch.exp2(extra["a_log2"][:s.state, :s.inner].double()), torch.exp(-torch.exp(m["A_log"])).T, rtol=1e-6)
    assert extra["a_log2"][s.state:].abs().sum() == 0 and torch.equal(extra["conv_w"][:, :s.inner].double(), m["conv"].T)


def test_state_sizes():
    for state in range(1, 257):
        p = SelectiveScan(inner=8, state=state, conv=2, dt_rank=3).state_p
        assert state <= p <= max(4, 1.6 * state) and any(p % n == 0 and p // n in (1, 2, 4, 8, 16) for n in (4, 8, 12, 16))


def test_cost_accounting_and_cache():
    cfg = CASES["wide"]
    model = meta_model(cfg, torch.bfloat16)
    weights_passed = sum(math.prod(s) for k, s in tensor_shapes(cfg).items() if len(s) == 2 and not k.endswith(("A_log", "conv")))
    assert model.num_active_matmul_params() == weights_passed                  # the embedding table counts once, as the output matrix
    per_token = 2 * (128 + 128) + 1 * (72 + 64)
    assert model.kv_bytes_per_token() == 2 * per_token
    scan = 2 * 256 * (16 + 3)
    states = scan + 2 * 2 * 128 * 64 + 2 * 256 * 200
    assert model.kv_read_bytes(10) == 10 * 2 * per_token + 4 * states
    assert model.kv_read_bytes(5000) == 2 * (38 * 2 * (128 + 128) + 202 * (72 + 64)) + 4 * states       # the window bounds what is read
    assert model.estimate_prefill_flops(8) > model.estimate_decode_flops(8) > 2 * model.num_active_matmul_params()
    mixers = model.run_mixers()
    assert [type(m).__name__ for m in mixers] == ["SelectiveScan", "WindowAttention", "Retention", "WindowAttention", "Retention"]
    cache = StackCache([m.row_width for m in mixers if m.cache == 0], [m.state_shape for m in mixers if m.cache == 1], torch.bfloat16, 2, 9, "cpu")
    assert [tuple(t.shape) for t in cache.rows] == [(2, 9, 512), (2, 9, 160)]        # (heads of 72 are padded to 96)
    assert [tuple(t.shape) for t in cache.states[0]] == [(2, 19, 256), (2, 2, 128, 64), (2, 1, 256, 256)]
    assert "SelectiveScan" in model.describe()


# ------------------------------------------------------------------------------------------------ the oracle's own checks
def test_oracle_lightning_is_the_quadratic_sum():
    m = pair(right_heads=3)["mixer"]["right"]
    w = {k: v.double() for k, v in ref.sub(weights(config([(pair(right_heads=3), None)])), "l0.mix.right.").items()}
    h = torch.randn(20, 96, dtype=torch.float64, generator=torch.Generator().manual_seed(0))
    got, _ = ref.lightning(h, w, m, 1e-5)
    H, dk, dv = m["heads"], m["dim"], m["vdim"]
    q, k, v = (torch.nn.functional.silu(h @ w[n].T).view(20, H, -1) for n in "qkv")
    o = torch.zeros(20, H, dv, dtype=torch.float64)
    for head, d in enumerate(m["decay"]):
        D = torch.tensor([[d ** (i - j) if j <= i else 0.0 for j in range(20)] for i in range(20)], dtype=torch.float64)
        o[:, head] = ((q[:, head] @ k[:, head].T) * D) @ v[:, head]
    o = o.reshape(20, -1)
    o = o / (o.pow(2).mean(-1, keepdim=True) + 1e-5).sqrt() * w["norm"]
    assert torch.allclose(got, (o * torch.sigmoid(h @ w["g"].T)) @ w["o"].T)


def test_oracle_attention_is_a_masked_softmax():
    c = pair()["mixer"]["left"]
    w = {k: v.double() for k, v in ref.sub(weights(config([(pair(), None)])), "l0.mix.left.").items()}
    T, H, G, dk, dv = 30, c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    h = torch.randn(T, 96, dtype=torch.float64, generator=torch.Generator().manual_seed(0))
    pos = torch.arange(T)[:, None]
    q, k = (ref.rotate(ref.rms_norm(h @ w[n].T + w[n + ".b"], 1e-5, w[n + ".norm"]).view(T, -1, dk), pos, c["rot"]) for n in "qk")
    v = (h @ w["v"].T + w["v.b"]).view(T, G, dv)
    k, v = k.repeat_interleave(H // G, 1), v.repeat_interleave(H // G, 1)
    i, j = torch.arange(T)[:, None], torch.arange(T)[None]
    s = torch.einsum("ihd,jhd->hij", q, k) * c["scale"]
    s = s.masked_fill(~((j <= i) & ((i - j < c["mask"]["size"]) | (j < c["mask"]["keep_first"]))), -math.inf)
    p = torch.softmax(torch.cat([s, w["sink"][:, None, None].expand(H, T, 1)], -1), -1)[..., :T]
    assert torch.allclose(ref.window_attention(h, w, c, 1e-5), torch.einsum("hij,jhd->ihd", p, v).reshape(T, -1) @ w["o"].T)


def test_oracle_scan_and_convolution():
    g = torch.Generator().manual_seed(1)
    x, dt, B, C = (torch.randn(12, n, dtype=torch.float64, generator=g) for n in (6, 6, 4, 4))
    dt, A, D = dt.exp(), -torch.rand(6, 4, dtype=torch.float64, generator=g), torch.randn(6, dtype=torch.float64, generator=g)
    y, end = ref.selective_scan(x, dt, A, B, C, D)
    at = dt.cumsum(0)
    for t in range(12):                         # the closed form: what token j put in, decayed by the steps since
        S = sum(torch.exp(A * (at[t] - at[j])[:, None]) * (dt[j] * x[j])[:, None] * B[j] for j in range(t + 1))
        assert torch.allclose(y[t], S @ C[t] + D * x[t])
    first, mid = ref.selective_scan(x[:5], dt[:5], A, B[:5], C[:5], D)
    rest, last = ref.selective_scan(x[5:], dt[5:], A, B[5:], C[5:], D, mid)
    assert torch.allclose(torch.cat([first, rest]), y) and torch.allclose(last, end)
    w, b = torch.randn(6, 3, dtype=torch.float64, generator=g), torch.randn(6, dtype=torch.float64, generator=g)
    want = torch.nn.functional.conv1d(torch.nn.functional.pad(x.T[None], (2, 0)), w[:, None], b, groups=6)[0].T
    assert torch.allclose(ref.causal_conv(x, w, b), want)


def test_oracle_is_causal_and_every_tensor_matters():
    cfg = CASES["odd"]
    w = {k: v.double() for k, v in weights(cfg).items()}
    toks = tokens(cfg, 30)
    full = ref.forward(cfg, w, toks)
    assert rel_rms(ref.forward(cfg, w, toks[:21]), full[:21]).max() < 1e-12
    g = torch.Generator().manual_seed(4)
    for name in w:
        noise = torch.randn(w[name].shape, generator=g, dtype=torch.float64) * w[name].std()
        assert rel_rms(ref.forward(cfg, dict(w, **{name: w[name] + noise}), toks), full).max() > 5e-3, name
