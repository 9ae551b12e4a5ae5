"""Synthetic stand-ins for what needs the network or a trained checkpoint: a model of a given depth with random
weights, and a tokenizer with the four methods the Engine uses.  Throughput does not depend on the weights."""
import torch

from .fp8 import convert_to_float8_training, fp8_module_filter
from .gpt import GPT, GPTConfig


def config_for_depth(depth, sequence_len=2048, vocab_size=32768, window_pattern="SSSL", aspect_ratio=64, head_dim=128,
                     n_kv_head=None):
    """The reference's depth -> shape rule (scripts/base_train.py:129-141): dim = depth * 64 rounded up to head_dim."""
    model_dim = -(-(depth * aspect_ratio) // head_dim) * head_dim
    n_head = model_dim // head_dim
    return GPTConfig(sequence_len=sequence_len, vocab_size=vocab_size, n_layer=depth, n_head=n_head,
                     n_kv_head=n_kv_head or n_head, n_embd=model_dim, window_pattern=window_pattern)


def random_init_model(cfg, device, seed=0):
    """Random weights drawn on the device with the distributions of the reference's init_weights (gpt.py:204-268), but
    with non-zero output projections, gates and lambdas so that every kernel does real work.  bf16, FP8 linears."""
    with torch.device("meta"):
        model = GPT(cfg)
    model.to_empty(device=device)
    g = torch.Generator(device=device).manual_seed(seed)
    s = 3 ** 0.5 * cfg.n_embd ** -0.5
    with torch.no_grad():
        for name, p in model.named_parameters():
            if name.endswith("wte.weight"):
                p.normal_(0.0, 0.8, generator=g)
            elif name == "lm_head.weight":
                p.normal_(0.0, 0.03, generator=g)
            elif "value_embeds" in name or "c_q" in name or "c_k" in name or "c_v" in name or "attn.c_proj" in name:
                p.uniform_(-s, s, generator=g)
            elif "c_fc" in name:
                p.uniform_(-0.4 * s, 0.4 * s, generator=g)
            elif "mlp.c_proj" in name:
                p.uniform_(-0.5 * s, 0.5 * s, generator=g)
            elif "gate" in name:
                p.uniform_(-0.5, 0.5, generator=g)
            elif name == "resid_lambdas":
                p.copy_(torch.linspace(1.15, 1.05, cfg.n_layer))
            elif name == "x0_lambdas":
                p.copy_(torch.linspace(0.20, 0.05, cfg.n_layer))
            elif name == "smear_lambda":
                p.fill_(0.35)
            elif name == "backout_lambda":
                p.fill_(0.2)
            else:
                raise RuntimeError(f"unhandled parameter {name}")
        model.to(torch.bfloat16)
    model.eval()
    convert_to_float8_training(model, module_filter_fn=fp8_module_filter)
    return model


def palilix_config(width, heads, rank=512, experts=64, top=6, expert_ff=1024, vocab=32768, groups=1, dense=False):
    """A Palilix configuration with the proportions of an ordinary model of this width: `groups` times (latent attention + dense,
    retention + experts twice, latent attention + experts), heads of 128, no repeated layers; `dense`: no experts."""
    head = width // heads
    moe = {"kind": "moe", "expert": {"ff": expert_ff, "limit": 7.0}, "router": {"experts": experts, "top": top}, "shared": {"ff": 2 * expert_ff, "limit": 7.0}}
    if dense:
        moe = {"kind": "dense", "ff": 4 * width - 64}        # (off the round number: no matrix has the shape of another's by accident)
    lat = {"heads": heads, "dim": head, "rot_dim": head // 2, "vdim": head, "kv_rank": rank, "scale": (1.5 * head) ** -0.5,
           "rot": {"base": 10000.0, "dims": head // 2}}
    ret = {"heads": heads, "dim": head, "vdim": head, "decay": [1 - 2.0 ** -(5 + 6 * i / max(1, heads - 1)) for i in range(heads)],
           "rot": {"base": 10000.0, "dims": head}}
    group = [{"type": "latent_attention", "mixer": lat, "mlp": moe if dense else {"kind": "dense", "ff": 4 * width}}, {"type": "retention", "mixer": ret, "mlp": moe},
             {"type": "retention", "mixer": ret, "mlp": moe}, {"type": "latent_attention", "mixer": lat, "mlp": moe}]
    return {"architecture": "Palilix", "embedding": {"scale": 1.0}, "layers": group * groups, "logit_scale": 1.0, "logit_softcap": 30.0,
            "norm": {"eps": 1e-6}, "vocab": vocab, "width": width}


def zodirax_config(width, heads, window=1024, vocab=32768, groups=1):
    """A Zodirax configuration with the proportions of an ordinary model of this width: `groups` times (window attention beside lightning
    attention, selective scan twice, the first again), heads of 128, four query heads per key head, SwiGLU of 8/3 of the width."""
    head = width // heads
    left = {"heads": heads, "kv_heads": max(1, heads // 4), "dim": head, "vdim": head, "scale": head ** -0.5, "mask": {"size": window, "keep_first": 4},
            "rot": {"base": 500000.0, "dims": head, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}}
    right = {"heads": heads, "dim": head, "vdim": head, "decay": [1 - 2.0 ** -(5 + 6 * i / max(1, heads - 1)) for i in range(heads)]}
    ff = {"kind": "dense", "ff": round(8 * width / 3 / 128) * 128}
    pair = {"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": 0.5, "right_scale": 0.5}, "mlp": ff}
    scan = {"type": "mamba1", "mixer": {"inner": 2 * width, "state": 16, "dt_rank": width // 16, "conv": 4}, "mlp": ff}
    return {"architecture": "Zodirax", "embedding": {"scale": 1.0}, "layers": [pair, scan, scan, pair] * groups, "norm": {"eps": 1e-6}, "vocab": vocab,
            "width": width}


def random_stack_model(cls, cfg, device, dtype=torch.bfloat16, seed=0):
    """A LayerStack design (its class and configuration) with random bf16 weights drawn on the device."""
    g = torch.Generator(device=device).manual_seed(seed)
    with torch.device("meta"):
        model = cls.from_config(cfg, dtype)
    tensors = {}
    for name, shape in model.tensor_shapes(model.config).items():
        t = torch.empty(shape, dtype=torch.bfloat16, device=device)
        if name == "embed" or name == "loop.step":
            t.normal_(0.0, 1.0, generator=g)
        elif name.endswith("A_log"):
            t.copy_(torch.arange(1, shape[1] + 1, device=device).log().expand(shape))
        elif name.endswith(".dt.b"):
            t.fill_(-4.0)
        elif len(shape) == 1:
            t.fill_(0.0 if model.config.norm_offset and "norm" in name and ".mix." not in name else 1.0)
        else:
            t.normal_(0.0, shape[-1] ** -0.5, generator=g)
        tensors[name] = t
    return model.load_tensors(tensors, device).eval()


class SyntheticTokenizer:
    """encode_special / get_bos_token_id / encode / decode: the Engine's whole view of a tokenizer (engine.py:186-192).
    The specials sit outside the vocabulary, so sampling from a random model never ends a row early."""

    def encode_special(self, s):
        return 1 << 30

    def get_bos_token_id(self):
        return (1 << 30) + 1

    def encode(self, s, prepend=None):
        return []

    def decode(self, tokens):
        return ""
