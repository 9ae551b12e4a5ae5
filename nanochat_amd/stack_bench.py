"""Prefill and decode throughput of the layer-stack designs at sizes like a real model's layers (random weights), with each kind of kernel
against its roofline: Palilix beside the FP8 GPT of equal width and number of layers (`bench.py --palilix`), Zodirax beside a Palilix of
dense layers and the GPT (`bench.py --zodirax`).

Rooflines: HBM 8 TB/s for kernels that stream weights, cached rows or states; the dense matrix peak of the operands' format (bf16 2.5,
fp8 5.0 PFLOP/s) for products of many rows.  Algorithmic bytes and flops: every weight, cached row and state once, visible pairs only, and
no credit for what a kernel repeats for exactness.  Kernel times are HIP event pairs around each launch.
"""
import ctypes as C
import time

import torch

from . import _lib
from .common import PEAK_BF16_FLOPS, PEAK_FP8_FLOPS, PEAK_HBM_BYTES_PER_S
from .engine import KVCache
from .gpt import GPTConfig
from .palilix import Palilix
from .stack import Experts, SelectiveScan
from .synthetic import palilix_config, random_init_model, random_stack_model, zodirax_config
from .zodirax import Zodirax

PREFILL = (1792,)
DECODE = (1, 16, 64)
CONTEXT = 2048
VOCAB = 32768


def _read(lib, cls):
    ms, units, n = C.c_double(), C.c_double(), C.c_int64()
    assert lib.nc_profile_read(cls, C.byref(ms), C.byref(units), C.byref(n)) == 0
    return ms.value, units.value, n.value


def _read_linear(lib, N, K):
    ms, units, n = C.c_double(), C.c_double(), C.c_int64()
    assert lib.nc_profile_read_gemm(N, K, C.byref(ms), C.byref(units), C.byref(n)) == 0
    return ms.value, units.value, n.value


def _timed(step, reps):
    for _ in range(3):
        step()
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(reps):
        step()
    torch.cuda.synchronize()
    return (time.perf_counter() - t0) / reps


def _profiled(lib, step, reps=4):
    step()
    torch.cuda.synchronize()
    lib.nc_profile_enable(1)
    for _ in range(reps):
        step()
    torch.cuda.synchronize()


def _entry(ms, units, n, peak, bound):
    if n == 0 or units == 0:
        return None
    rate = units / (ms * 1e-3)
    return {"launches": n, "us": round(ms * 1e3 / n, 2), "bound": bound, "rate": round(rate / 1e12, 3), "unit": "TB/s" if bound == "hbm" else "TFLOP/s",
            "frac": round(rate / peak, 4)}


def _linears(lib, shapes, decode, peak, weight_bytes):
    """One entry per weight shape: streamed bytes at decode, flops at prefill."""
    out = {}
    for name, (N, K, flops_rows) in shapes.items():
        ms, _, n = _read_linear(lib, N, K)
        units = n * (N * K * weight_bytes if decode else 2.0 * flops_rows * N * K)
        e = _entry(ms, units, n, PEAK_HBM_BYTES_PER_S if decode else peak, "hbm" if decode else "mfma")
        if e:
            out[name] = e
    return out


def _stack_shapes(sc, Wp):
    """{names: (N, K)} of the weights of a stack's layers; weights of one shape are one entry."""
    shapes = {}

    def add(name, N, K):
        names = shapes.setdefault((N, K), [])
        if name not in names:
            names.append(name)
    for layer in sc.layers:
        f, kind = layer.ff, "+".join(type(m).__name__ for m in layer.mixers)
        n_in, k_out = sum(m.cols for m in layer.mixers), sum(m.out for m in layer.mixers)
        if f is not None and sc.block == "post_norm":
            add(f"{type(f).__name__} in", f.ff_cols, Wp)
            add(f"{type(f).__name__} out", Wp, f.ff_p)
        elif f is not None:
            kind += f"+{type(f).__name__}"
            n_in, k_out = n_in + f.router_cols + f.ff_cols, k_out + f.ff_p
        add(f"{kind} in", n_in, Wp)
        add(f"{kind} out", Wp, k_out)
        for m in layer.mixers:
            if isinstance(m, SelectiveScan):
                add("scan x", m.dt_rank_p + 2 * m.bc_p, m.inner_p)
                add("scan dt", m.inner_p, m.dt_rank_p)
    return {" / ".join(names): shape for shape, names in shapes.items()}


# timing class of the library -> (name, bound of a prompt, bound of decoding)
STACK_CLASSES = {0: ("latent attention", "mfma", "hbm"), 2: ("retention", "hbm", "hbm"), 5: ("window attention", "mfma", "hbm"), 6: ("selective scan", "hbm", "hbm")}


def bench_stack(cls, cfg, device):
    model = random_stack_model(cls, cfg, device)
    lib = _lib.stack_lib()
    sc, Wp = model.config, model.width_p
    g = torch.Generator(device=device).manual_seed(1)

    def kernels(rows, decode):
        shapes = {name: (N, K, rows) for name, (N, K) in _stack_shapes(sc, Wp).items()}
        if decode:
            shapes["head"] = (VOCAB, Wp, rows)          # (a prompt has one row of logits)
        out = _linears(lib, shapes, decode, PEAK_BF16_FLOPS, 2)
        for c, (name, prompt, single) in STACK_CLASSES.items():
            bound = single if decode else prompt
            out[name] = _entry(*_read(lib, c), PEAK_HBM_BYTES_PER_S if bound == "hbm" else PEAK_BF16_FLOPS, bound)
        ff = next((l.ff for l in sc.layers if isinstance(l.ff, Experts)), None)
        if ff is not None:
            ms, units, n = _read(lib, 4)
            # how many experts a step touches, on average, if every choice is as likely
            touched = ff.experts * (1 - (1 - ff.top / ff.experts) ** rows)
            out["experts"] = _entry(ms, n / 2 * touched * 3 * ff.expert_ff_p * Wp * 2 if decode else units, n, PEAK_HBM_BYTES_PER_S if decode else PEAK_BF16_FLOPS,
                                    "hbm" if decode else "mfma")
        out["row kernels ms per step"] = round(_read(lib, 3)[0] / 4, 4)
        lib.nc_profile_enable(0)
        return {k: v for k, v in out.items() if v is not None}

    res = {"layers": len(sc.layers), "width": cfg["width"], "parameters": sum(p.numel() for p in model.parameters()), "prefill": {}, "decode": {}}
    for T in PREFILL:
        ids = torch.randint(0, VOCAB, (1, T), device=device, generator=g)
        cache = model.new_cache(1, T)

        def step():
            cache.reset()
            model.forward_last(ids, kv_cache=cache)
        s = _timed(step, 10)
        _profiled(lib, step)
        res["prefill"][T] = {"ms": round(s * 1e3, 3), "tokens_per_s": round(T / s, 1), "kernels": kernels(T, False)}
    for B in DECODE:
        cache = model.new_cache(B, CONTEXT + 64)
        for t in cache.rows:
            t.normal_(generator=g)
        cache.cache_seqlens.fill_(CONTEXT - 32)
        cache._host_pos = [CONTEXT - 32] * B
        cache._positions_changed()
        tok = torch.randint(0, VOCAB, (B, 1), device=device, generator=g)
        s = _timed(lambda: model.forward_last(tok, kv_cache=cache), 30)
        _profiled(lib, lambda: model.forward_last(tok, kv_cache=cache))
        res["decode"][B] = {"ms": round(s * 1e3, 4), "tokens_per_s": round(B / s, 1), "kernels": kernels(B, True)}
        del cache
    return res


def bench_gpt(width, device, layers):
    H = width // 128
    model = random_init_model(GPTConfig(sequence_len=CONTEXT + 64, vocab_size=VOCAB, n_layer=layers, n_head=H, n_kv_head=H, n_embd=width, window_pattern="L"),
                              device)
    lib = _lib.lib()
    g = torch.Generator(device=device).manual_seed(1)

    def kernels(rows, decode, keys):
        E = width
        shapes = {"qkv": (3 * E, E, rows), "attention out": (E, H * 128, rows), "mlp in": (4 * E, E, rows), "mlp out": (E, 4 * E, rows)}
        if decode:
            shapes["head"] = (VOCAB, E, rows)
        out = _linears(lib, shapes, decode, PEAK_FP8_FLOPS, 1)
        ms, _, n = _read(lib, 0)
        units = n * (rows * keys * 2 * H * 128 * 2 if decode else 4.0 * H * 128 * rows * (rows + 1) / 2)
        out["attention"] = _entry(ms, units, n, PEAK_HBM_BYTES_PER_S if decode else PEAK_BF16_FLOPS, "hbm" if decode else "mfma")
        out["row kernels ms per step"] = round((_read(lib, 3)[0] + _read(lib, 2)[0]) / 4, 4)
        lib.nc_profile_enable(0)
        return {k: v for k, v in out.items() if v is not None}

    res = {"layers": layers, "width": width, "parameters": sum(p.numel() for p in model.parameters()), "prefill": {}, "decode": {}}
    for T in PREFILL:
        ids = torch.randint(0, VOCAB, (1, T), device=device, generator=g)
        cache = KVCache(1, H, T, 128, layers, device, torch.bfloat16)

        def step():
            cache.reset()
            model.forward_last(ids, kv_cache=cache)
        s = _timed(step, 10)
        _profiled(lib, step)
        res["prefill"][T] = {"ms": round(s * 1e3, 3), "tokens_per_s": round(T / s, 1), "kernels": kernels(T, False, T)}
    for B in DECODE:
        cache = KVCache(B, H, CONTEXT + 64, 128, layers, device, torch.bfloat16)
        cache.k_cache.normal_(generator=g)
        cache.v_cache.normal_(generator=g)
        cache.set_seqlens([CONTEXT - 32] * B)
        cache.prev_embedding = torch.randn(B, 1, width, device=device, generator=g).bfloat16()
        tok = torch.randint(0, VOCAB, (B, 1), device=device, generator=g)
        s = _timed(lambda: model.forward_last(tok, kv_cache=cache), 30)
        _profiled(lib, lambda: model.forward_last(tok, kv_cache=cache))
        res["decode"][B] = {"ms": round(s * 1e3, 4), "tokens_per_s": round(B / s, 1), "kernels": kernels(B, True, CONTEXT + 4)}
        del cache
    return res


def _groups(width):
    return 2 if width <= 2048 else 1


def run_palilix(device, widths=(2048, 4096)):
    out = {}
    for width in widths:
        p = bench_stack(Palilix, palilix_config(width, width // 128, vocab=VOCAB, groups=_groups(width)), device)
        torch.cuda.empty_cache()
        out[f"width {width}"] = {"palilix": p, "gpt": bench_gpt(width, device, p["layers"])}
        torch.cuda.empty_cache()
    return out


def run_zodirax(device, widths=(2048, 4096)):
    out = {}
    for width in widths:
        z = bench_stack(Zodirax, zodirax_config(width, width // 128, vocab=VOCAB, groups=_groups(width)), device)
        torch.cuda.empty_cache()
        p = bench_stack(Palilix, palilix_config(width, width // 128, vocab=VOCAB, groups=_groups(width), dense=True), device)
        torch.cuda.empty_cache()
        out[f"width {width}"] = {"zodirax": z, "palilix, dense": p, "gpt": bench_gpt(width, device, z["layers"])}
        torch.cuda.empty_cache()
    return out
