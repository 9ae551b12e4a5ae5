"""What the GPU tests of the layer-stack designs share: running one sequence in portions, judging logits against the oracle's, writing a
model folder, loading the trace runner."""
import importlib.machinery
import importlib.util
import json
import os
import struct

import torch

DEV = "cuda"
DTYPES = [torch.float32, torch.bfloat16]
# difference from the oracle per position (root mean square over the vocabulary, relative): 32-bit rounding, bf16 rounding
BAR = {torch.float32: 2e-5, torch.bfloat16: 4e-2}


def say(msg):
    print(f"[gpu-case] {msg}", flush=True)


def build_model(cls, cfg, w, dtype):
    with torch.device("meta"):
        model = cls.from_config(cfg, dtype)
    return model.load_tensors(w, DEV)


def ids(toks):
    return torch.tensor([toks], dtype=torch.long, device=DEV)


def tokens(cfg, n, seed=1):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def rel_rms(got, want):
    """Per position: root mean square of the difference over that of the (centred) logits."""
    got, want = got.double().cpu(), want.double()
    scale = (want - want.mean(-1, keepdim=True)).pow(2).mean().sqrt()
    return ((got - want).pow(2).mean(-1).sqrt() / scale)


def run(model, toks, cuts, seq_len=None):
    """Logits [T, vocab] of one sequence brought in portions of the given sizes."""
    cache = model.new_cache(1, seq_len or len(toks))
    out, at = [], 0
    for n in cuts:
        out.append(model.forward(ids(toks[at:at + n]), kv_cache=cache)[0].clone())
        at += n
    assert at == len(toks) == cache.get_pos() == int(cache.cache_seqlens[0])
    return torch.cat(out)


def judge(err, dtype, what, bar=None):
    """Every position below the bar in 32-bit.  In bf16 one position in thirty (or one) may lie over it, up to ten times: where two experts
    score almost alike, or a head's output is almost zero before its norm, a rounded input turns into another answer."""
    bar = bar or BAR[dtype]
    worst, over = err.max().item(), int((err > bar).sum())
    print(f"{what} {str(dtype)[6:]}: worst position {worst:.2e}, {over} of {err.numel()} over {bar:.0e}", flush=True)
    allowed = 0 if dtype == torch.float32 else max(1, err.numel() // 30)
    assert worst == worst and over <= allowed and worst <= (bar if allowed == 0 else 10 * bar), f"{what}: worst at {err.argmax().item()}"


def check(got, want, dtype, what, bar=None):
    judge(rel_rms(got, want), dtype, what, bar)


def write_model(path, cfg, w):
    blob, header = b"", {}
    for k, t in w.items():
        data = t.contiguous().view(torch.int16).numpy().tobytes()
        header[k] = {"dtype": "BF16", "shape": list(t.shape), "data_offsets": [len(blob), len(blob) + len(data)]}
        blob += data
    head = json.dumps(header).encode()
    (path / "model.safetensors").write_bytes(struct.pack("<Q", len(head)) + head + blob)
    (path / "config.json").write_text(json.dumps(cfg))


def trace_runner():
    """bin/trace_run as a module."""
    path = os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "bin", "trace_run")
    loader = importlib.machinery.SourceFileLoader("trace_run", path)
    mod = importlib.util.module_from_spec(importlib.util.spec_from_loader("trace_run", loader))
    loader.exec_module(mod)
    return mod
