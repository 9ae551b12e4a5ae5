"""Decoders made of configured layers: any order of mixers and feed-forwards, a run of layers that may repeat with the same weights.

A layer is `x += mixer(h) + ff(h)` with `h = layer_norm(x)`.  The mechanisms are classes of their own with their sizes and constants as
fields; each knows the tensors it needs, how they are packed for the kernels and what it keeps per sequence:

    mixers         LatentAttention, Retention
    feed-forwards  DenseGelu, Experts (clamped GLU experts, softmax router, optional shared expert)

`LayerStack` is the model: weights by name, a packed plan that is rebuilt whenever a weight changes, and a forward that is one native
call (nc_stack_forward).  It has the surface the Engine and the harness use on every model of this package (forward, forward_last,
new_cache, get_device, the cost accounting).  A design is a class that turns its configuration into a StackConfig (palilix.py).

Two storage types: bfloat16 (matrix products in bf16 with 32-bit sums; residual stream, norms, angles, scores, router and recurrent
state in 32-bit), and float32 (everything in true 32-bit).
"""
import ctypes as C
import math
from dataclasses import dataclass, field

import torch
import torch.nn as nn

from . import _lib, ops

PAD = ops.STACK_PAD


def round_up(n, m):
    return -(-n // m) * m


def padded(t, *shape):
    """t in the leading corner of a zero tensor of `shape`."""
    out = torch.zeros(shape, dtype=t.dtype, device=t.device)
    out[tuple(slice(0, n) for n in t.shape)] = t
    return out


# ------------------------------------------------------------------------------------------------ mixers
@dataclass
class LatentAttention:
    """Causal softmax attention whose keys and values are linear in one cached latent per token, plus one rotated key part that the heads
    share.  Per head: `dim` unrotated and `rot_dim` rotated query / key dimensions, `vdim` values; the latent has `rank` values."""
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    rank: int
    scale: float
    rot_base: float

    kind = 0

    def __post_init__(self):
        assert self.rot_dim % 2 == 0, f"rotated part of odd size {self.rot_dim}"
        self.rot_dims = self.rot_dim
        self.dim_p, self.rot_p, self.rank_p = round_up(self.dim, 32), round_up(self.rot_dim, 32), round_up(self.rank, PAD)
        # the heads' values side by side fill whole K-steps of the output matrix
        self.vdim_p = round_up(self.vdim, 16 * (4 // math.gcd(self.heads, 4)))
        self.mix_cols = self.heads * (self.dim_p + self.rot_p) + self.rank_p + self.rot_p
        self.mix_out = self.heads * self.vdim_p
        self.latent_width = self.rank_p + self.rot_p

    def tensors(self, width):
        H = self.heads
        return {"q": (H * (self.dim + self.rot_dim), width), "dkv": (self.rank + self.rot_dim, width), "dkv.norm": (self.rank,),
                "uk": (H * self.dim, self.rank), "uv": (H * self.vdim, self.rank), "o": (width, H * self.vdim)}

    def pack(self, w):
        """(rows of the input matrix, columns of the output matrix, further tensors of the descriptor)."""
        H, width = self.heads, w["q"].shape[1]
        q = torch.zeros(H, self.dim_p + self.rot_p, width, dtype=w["q"].dtype, device=w["q"].device)
        parts = w["q"].view(H, self.dim + self.rot_dim, width)
        q[:, :self.dim], q[:, self.dim_p:self.dim_p + self.rot_dim] = parts[:, :self.dim], parts[:, self.dim:]
        dkv = torch.zeros(self.rank_p + self.rot_p, width, dtype=q.dtype, device=q.device)
        dkv[:self.rank], dkv[self.rank_p:self.rank_p + self.rot_dim] = w["dkv"][:self.rank], w["dkv"][self.rank:]
        uk, uv = w["uk"].view(H, self.dim, self.rank), w["uv"].view(H, self.vdim, self.rank)
        ukv = torch.zeros(H, self.dim_p + self.vdim_p, self.rank_p, dtype=q.dtype, device=q.device)
        ukv[:, :self.dim, :self.rank], ukv[:, self.dim_p:self.dim_p + self.vdim, :self.rank] = uk, uv
        o = padded(w["o"].view(width, H, self.vdim), width, H, self.vdim_p).view(width, H * self.vdim_p)
        return (torch.cat([q.view(-1, width), dkv]), o,
                {"kv_norm_w": padded(w["dkv.norm"].float(), self.rank_p), "w_uk_t": padded(uk.transpose(1, 2), H, self.rank_p, self.dim_p), "w_ukv": ukv})

    def describe(self, d):
        d.dim, d.dim_p, d.vdim, d.vdim_p, d.rot_dim, d.rot_p, d.rot_dims = (self.dim, self.dim_p, self.vdim, self.vdim_p, self.rot_dim, self.rot_p,
                                                                              self.rot_dims)
        d.rank, d.rank_p, d.score_scale = self.rank, self.rank_p, self.scale

    def flops(self, keys):
        """Of one token that sees `keys` keys, beyond its projections: the latent-space form."""
        return 2 * self.heads * (self.rank * (self.dim + self.vdim) + keys * (2 * self.rank + self.rot_dim))

    def prefill_flops(self, tokens):
        """The expanded form: keys and values of every token, then causal pairs."""
        return 2 * self.heads * (tokens * self.rank * (self.dim + self.vdim) + tokens * (tokens + 1) // 2 * (self.dim + self.rot_dim + self.vdim))

    def read_elements(self, keys):
        """(storage-type elements, fp32 elements) of cache a token reads or writes."""
        return keys * (self.rank + self.rot_dim), 0


@dataclass
class Retention:
    """Linear attention with one fixed decay per head, rotary positions on the first `rot_dims` dimensions of q and k, outputs normed per
    head and gated.  `decay` holds one factor per head."""
    heads: int
    dim: int
    vdim: int
    decay: list
    rot_dims: int
    rot_base: float
    k_scale: float = field(default=None)

    kind = 1

    def __post_init__(self):
        assert len(self.decay) == self.heads, f"{len(self.decay)} decays for {self.heads} heads"
        assert self.rot_dims % 2 == 0 and self.rot_dims <= self.dim
        if self.k_scale is None:
            self.k_scale = self.dim ** -0.5
        # sizes the kernels hold a state in registers for; larger ones go through memory
        sizes = [n for n in (64, 128, 256)]
        self.dim_p = next((n for n in sizes if n >= self.dim), round_up(self.dim, PAD))
        self.vdim_p = next((n for n in sizes if n >= max(self.vdim, 128 if self.dim_p == 256 else 0)), round_up(self.vdim, PAD))
        self.mix_cols = 2 * self.heads * (self.dim_p + self.vdim_p)
        self.mix_out = self.heads * self.vdim_p
        self.state_shape = (self.heads, self.dim_p, self.vdim_p)

    def tensors(self, width):
        H = self.heads
        return {"q": (H * self.dim, width), "k": (H * self.dim, width), "v": (H * self.vdim, width), "g": (H * self.vdim, width),
                "o": (width, H * self.vdim)}

    def pack(self, w):
        H, width = self.heads, w["q"].shape[1]

        def heads(t, n, n_p):
            return padded(t.view(H, n, width), H, n_p, width).view(H * n_p, width)
        rows = [heads(w["q"], self.dim, self.dim_p), heads(w["k"], self.dim, self.dim_p), heads(w["v"], self.vdim, self.vdim_p),
                heads(w["g"], self.vdim, self.vdim_p)]
        o = padded(w["o"].view(width, H, self.vdim), width, H, self.vdim_p).view(width, H * self.vdim_p)
        decay = torch.tensor(self.decay, dtype=torch.float32)
        log2 = torch.log2(decay.double()).clamp(min=-1000.0).float()          # a decay of 0 forgets everything: 2^-1000 is 0 as well
        return torch.cat(rows), o, {"decay": torch.stack([decay, log2], dim=1).to(o.device)}

    def describe(self, d):
        d.dim, d.dim_p, d.vdim, d.vdim_p, d.rot_dims, d.score_scale = self.dim, self.dim_p, self.vdim, self.vdim_p, self.rot_dims, self.k_scale

    def flops(self, keys):
        return 4 * self.heads * self.dim * self.vdim

    def prefill_flops(self, tokens):
        return tokens * self.flops(0)

    def read_elements(self, keys):
        return 0, 2 * self.heads * self.dim * self.vdim


# ------------------------------------------------------------------------------------------------ feed-forwards
def interleaved(gate, up, rows_p, cols_p):
    """gate and up row by row, zero rows and columns behind: their product's neighbouring columns belong together."""
    both = torch.stack([padded(gate, rows_p, cols_p), padded(up, rows_p, cols_p)], dim=1)
    return both.view(2 * rows_p, cols_p)


@dataclass
class DenseGelu:
    """down gelu(up h), tanh form."""
    ff: int

    kind = 1

    def __post_init__(self):
        self.ff_p = round_up(self.ff, PAD)
        self.router_cols, self.ff_cols = 0, self.ff_p

    def tensors(self, width):
        return {"up": (self.ff, width), "down": (width, self.ff)}

    def pack(self, w, width_p):
        return None, padded(w["up"], self.ff_p, width_p), padded(w["down"], width_p, self.ff_p), {}

    def describe(self, d):
        d.ff_limit = 0.0

    def active_params(self, width):
        return 2 * self.ff * width


@dataclass
class Experts:
    """`experts` clamped GLU layers of which a token uses the `top` that a softmax router scores highest, weighted by their scores over
    the chosen scores' sum; a shared expert of its own size, if any, runs for every token."""
    experts: int
    top: int
    ff: int
    limit: float
    shared_ff: int = 0
    shared_limit: float = 0.0

    kind = 2

    def __post_init__(self):
        assert 1 <= self.top <= self.experts
        self.expert_ff_p, self.ff_p = round_up(self.ff, PAD), round_up(self.shared_ff, PAD)
        self.router_cols, self.ff_cols = round_up(self.experts, 16), 2 * self.ff_p

    def tensors(self, width):
        out = {"router": (self.experts, width)}
        for name, n in [(f"e{i}", self.ff) for i in range(self.experts)] + ([("shared", self.shared_ff)] if self.shared_ff else []):
            out |= {f"{name}.gate": (n, width), f"{name}.up": (n, width), f"{name}.down": (width, n)}
        return out

    def stacked(self):
        """{name of one parameter: the tensors it holds, one per expert}."""
        return {f"experts.{part}": [f"e{i}.{part}" for i in range(self.experts)] for part in ("gate", "up", "down")}

    def pack(self, w, width_p):
        router = padded(w["router"], self.router_cols, width_p)
        e1 = torch.empty(self.experts, 2 * self.expert_ff_p, width_p, dtype=router.dtype, device=router.device)
        for i in range(self.experts):
            e1[i] = interleaved(w["experts.gate"][i], w["experts.up"][i], self.expert_ff_p, width_p)
        e2 = padded(w["experts.down"], self.experts, width_p, self.expert_ff_p)
        first = last = None
        if self.shared_ff:
            first = interleaved(w["shared.gate"], w["shared.up"], self.ff_p, width_p)
            last = padded(w["shared.down"], width_p, self.ff_p)
        return router, first, last, {"w_e1": e1, "w_e2": e2}

    def describe(self, d):
        d.experts, d.top, d.expert_ff_p, d.expert_limit, d.ff_limit = self.experts, self.top, self.expert_ff_p, self.limit, self.shared_limit

    def active_params(self, width):
        return width * (self.experts + 3 * self.top * self.ff + 3 * self.shared_ff)


# ------------------------------------------------------------------------------------------------ configuration
@dataclass
class LayerSpec:
    mixer: object
    ff: object = None               # None: no feed-forward


@dataclass
class StackConfig:
    vocab_size: int
    n_embd: int
    layers: list                    # LayerSpec
    eps: float
    embed_scale: float = 1.0
    logit_scale: float = 1.0
    logit_softcap: float = 0.0      # 0: none
    loop_start: int = 0             # layers [loop_start, loop_stop) run loop_times times
    loop_stop: int = 0
    loop_times: int = 1
    loop_steps: bool = False        # a learned vector is added at the start of every pass
    sequence_len: int = 2048        # how far a generation without a token limit goes; the model itself has no limit

    @property
    def n_layer(self):
        return len(self.layers)

    def runs(self):
        """[(layer, add the embedding output first, step vector to add first or -1)] in the order the layers run."""
        if not (0 <= self.loop_start <= self.loop_stop <= len(self.layers) and self.loop_times >= 1):
            raise ValueError(f"loop over layers {self.loop_start}..{self.loop_stop} x {self.loop_times} of {len(self.layers)}")
        out = [(i, False, -1) for i in range(self.loop_start)]
        for t in range(self.loop_times):
            for i in range(self.loop_start, self.loop_stop):
                first = i == self.loop_start
                out.append((i, first and t > 0, t if first and self.loop_steps else -1))
        return out + [(i, False, -1) for i in range(self.loop_stop, len(self.layers))]


# ------------------------------------------------------------------------------------------------ the model
class LayerStack(nn.Module):
    WORKSPACE_CACHE_BYTES = 4 << 30       # step workspaces kept alive between calls (one per shape seen)

    def __init__(self, config, dtype=torch.bfloat16):
        super().__init__()
        if dtype not in ops.STACK_DTYPES:
            raise ValueError(f"a layer stack runs in bfloat16 or float32, not {dtype}")
        self.config = config
        self.dtype = dtype
        self.width_p = round_up(config.n_embd, PAD)
        self.run_list = config.runs()
        # parameters under their tensor names ('.' is not allowed in a parameter's name); an expert layer's tensors of one kind are one
        # parameter, with one row of it per tensor
        shapes = self.tensor_shapes(config)
        self._stacks = {f"l{i}.mlp.{k}": [f"l{i}.mlp.{n}" for n in names] for i, layer in enumerate(config.layers) if isinstance(layer.ff, Experts)
                        for k, names in layer.ff.stacked().items()}
        inside = {n for names in self._stacks.values() for n in names}
        held = {k: s for k, s in shapes.items() if k not in inside} | {k: (len(names), *shapes[names[0]]) for k, names in self._stacks.items()}
        self.tensors = nn.ParameterDict({k.replace(".", "/"): nn.Parameter(torch.empty(s), requires_grad=False) for k, s in held.items()})
        self._plan = None
        self._plan_key = None
        self._rope = {}
        self._rope_len = 0
        self._workspaces = {}

    @staticmethod
    def tensor_shapes(config):
        """{tensor name: shape} of the whole model."""
        W = config.n_embd
        out = {"embed": (config.vocab_size, W)}
        if config.loop_steps:
            out["loop.step"] = (config.loop_times, W)
        for i, layer in enumerate(config.layers):
            out[f"l{i}.norm1"] = (W,)
            out |= {f"l{i}.mix.{k}": s for k, s in layer.mixer.tensors(W).items()}
            if layer.ff is not None:
                out |= {f"l{i}.mlp.{k}": s for k, s in layer.ff.tensors(W).items()}
        return out | {"final.norm": (W,), "head": (config.vocab_size, W)}

    def held_tensors(self):
        """{name: parameter} as the model holds them (experts of a layer together)."""
        return {k.replace("/", "."): p for k, p in self.tensors.items()}

    def named_tensors(self):
        """{tensor name: tensor} as in a weight file; an expert's is a view of its layer's parameter."""
        out = {}
        for name, p in self.held_tensors().items():
            out |= dict(zip(self._stacks[name], p.unbind(0))) if name in self._stacks else {name: p}
        return out

    def load_tensors(self, tensors, device):
        """Take the weights by name, in the dtype they come in; names and shapes must be exactly the model's."""
        want = self.tensor_shapes(self.config)
        missing, extra = sorted(set(want) - set(tensors)), sorted(set(tensors) - set(want))
        if missing or extra:
            raise RuntimeError(f"weights do not match the model: missing {missing[:4]}, unexpected {extra[:4]}")
        for name, shape in want.items():
            if tuple(tensors[name].shape) != tuple(shape):
                raise RuntimeError(f"{name}: shape {tuple(tensors[name].shape)} in the file, {tuple(shape)} in the model")
        for name in self.held_tensors():
            t = torch.stack([tensors[n] for n in self._stacks[name]]) if name in self._stacks else tensors[name]
            self.tensors[name.replace(".", "/")] = nn.Parameter(t.to(device), requires_grad=False)
        self.invalidate_plan()
        return self

    def get_device(self):
        return self.tensors["embed"].device

    def invalidate_plan(self):
        self._plan = None

    def _apply(self, fn, recurse=True):
        self.invalidate_plan()
        return super()._apply(fn, recurse)

    # ---- cache
    def new_cache(self, batch_size, seq_len, prefill_from=None, share_prompt_reads=False):
        """(share_prompt_reads: every model's new_cache takes it; latents are read per row here)"""
        from .engine import StackCache
        mixers = [self.config.layers[i].mixer for i, _, _ in self.run_list]
        cache = StackCache([m.latent_width for m in mixers if isinstance(m, LatentAttention)], [m.state_shape for m in mixers if isinstance(m, Retention)],
                           self.dtype, batch_size, seq_len, self.get_device(), prefill_from=prefill_from)
        return cache

    # ---- cost accounting
    def num_active_matmul_params(self):
        """Weights a token is multiplied with, over all layer runs and the output matrix."""
        W, total = self.config.n_embd, self.config.vocab_size * self.config.n_embd
        for i, _, _ in self.run_list:
            layer = self.config.layers[i]
            skip = ("uk", "uv", "dkv.norm")      # applied per key or query: in the mixer's own count
            total += sum(math.prod(s) for k, s in layer.mixer.tensors(W).items() if k not in skip)
            total += layer.ff.active_params(W) if layer.ff is not None else 0
        return total

    def estimate_decode_flops(self, context_len):
        return 2 * self.num_active_matmul_params() + sum(self.config.layers[i].mixer.flops(context_len) for i, _, _ in self.run_list)

    def estimate_prefill_flops(self, num_tokens):
        return 2 * self.num_active_matmul_params() * num_tokens + sum(self.config.layers[i].mixer.prefill_flops(num_tokens) for i, _, _ in self.run_list)

    def kv_bytes_per_token(self):
        """Cache bytes that grow with the sequence (a recurrent state does not)."""
        es = self.dtype.itemsize
        return sum(self.config.layers[i].mixer.read_elements(1)[0] for i, _, _ in self.run_list) * es

    def kv_read_bytes(self, context_len):
        """Cache bytes one decode step reads or writes per row."""
        parts = [self.config.layers[i].mixer.read_elements(context_len) for i, _, _ in self.run_list]
        return sum(p[0] for p in parts) * self.dtype.itemsize + sum(p[1] for p in parts) * 4

    def streamed_weight_bytes(self):
        """Weight bytes one single-row decode step reads."""
        per_head = sum(math.prod(s) for i, _, _ in self.run_list for k, s in self.config.layers[i].mixer.tensors(self.config.n_embd).items() if k in ("uk", "uv"))
        return (self.num_active_matmul_params() + per_head) * self.dtype.itemsize

    def describe(self):
        kinds = [type(layer.mixer).__name__ for layer in self.config.layers]
        mix = ", ".join(f"{kinds.count(k)} {k}" for k in dict.fromkeys(kinds))
        return f"layers {len(kinds)} ({mix}), {len(self.run_list)} layer runs, dim {self.config.n_embd}"

    # ---- plan
    def _rope_table(self, base, dims):
        """cos, sin of position * base^(-2i/dims), fp32 [len, dims/2, 2] (worked out in fp64: an angle of thousands of radians keeps its
        fraction)."""
        key = (base, dims)
        t = self._rope.get(key)
        if t is None:
            dev = self.get_device()
            i = torch.arange(dims // 2, dtype=torch.float64, device=dev)
            ang = torch.outer(torch.arange(self._rope_len, dtype=torch.float64, device=dev), base ** (-2.0 * i / max(dims, 1)))
            t = self._rope[key] = torch.stack([ang.cos(), ang.sin()], dim=-1).float().contiguous()
        return t

    def _build_plan(self):
        cfg, Wp = self.config, self.width_p
        dev = self.get_device()
        if dev.type != "cuda":
            raise RuntimeError("the layer stack runs on the GPU only: load the model on cuda (there is no CPU fallback)")
        w = {k: p.detach() for k, p in self.held_tensors().items()}
        keep = []

        def own(t, dtype):
            t = t.to(dtype).contiguous()
            keep.append(t)
            return t.data_ptr()

        layers = (_lib.StackLayer * cfg.n_layer)()
        for i, spec in enumerate(cfg.layers):
            d, mixer, ff = layers[i], spec.mixer, spec.ff
            pick = lambda prefix: {k[len(prefix):]: v.to(self.dtype) if v.dim() > 1 else v for k, v in w.items() if k.startswith(prefix)}  # noqa: E731
            rows, cols, extra = mixer.pack(pick(f"l{i}.mix."))
            rows, cols = [padded(rows, rows.shape[0], Wp)], [padded(cols, Wp, mixer.mix_out)]
            d.mixer, d.heads, d.mix_cols, d.mix_out = mixer.kind, mixer.heads, mixer.mix_cols, mixer.mix_out
            mixer.describe(d)
            if ff is not None:
                router, first, last, more = ff.pack(pick(f"l{i}.mlp."), Wp)
                rows += [t for t in (router, first) if t is not None]
                cols += [t for t in (last,) if t is not None]
                extra |= more
                d.ff, d.router_cols, d.ff_cols, d.ff_p = ff.kind, ff.router_cols, ff.ff_cols, ff.ff_p
                ff.describe(d)
            d.n_in, d.k_out = d.mix_cols + d.router_cols + d.ff_cols, d.mix_out + d.ff_p
            d.w_in, d.w_out = own(torch.cat(rows), self.dtype), own(torch.cat(cols, dim=1), self.dtype)
            d.norm_w = own(padded(w[f"l{i}.norm1"].float(), Wp), torch.float32)
            for name, t in extra.items():
                setattr(d, name, own(t, torch.float32 if name in ("kv_norm_w", "decay") else self.dtype))
        runs = (_lib.StackRun * len(self.run_list))()
        used = {0: 0, 1: 0}
        for r, (i, again, step) in zip(runs, self.run_list):
            kind = cfg.layers[i].mixer.kind
            r.layer, r.slot, r.add_embedding, r.step = i, used[kind], int(again), step
            used[kind] += 1
        md = _lib.StackModel()
        md.dtype, md.width, md.width_p, md.vocab = ops.STACK_DTYPES[self.dtype], cfg.n_embd, Wp, cfg.vocab_size
        md.n_layers, md.n_runs, md.max_k_out = cfg.n_layer, len(self.run_list), max(d.k_out for d in layers)
        md.eps, md.embed_scale, md.logit_scale, md.logit_softcap = cfg.eps, cfg.embed_scale, cfg.logit_scale, cfg.logit_softcap
        md.embed = own(padded(w["embed"], cfg.vocab_size, Wp), self.dtype)
        md.head = own(padded(w["head"], cfg.vocab_size, Wp), self.dtype)
        md.final_norm_w = own(padded(w["final.norm"].float(), Wp), torch.float32)
        if cfg.loop_steps:
            md.steps = own(padded(w["loop.step"].float(), cfg.loop_times, Wp), torch.float32)
        md.layers, md.runs = C.cast(layers, C.POINTER(_lib.StackLayer)), C.cast(runs, C.POINTER(_lib.StackRun))
        self._plan = (md, layers, runs, keep)
        self._rope_len = 0                       # the tables go with the plan (device, layers)
        self._workspaces = {}

    def _ensure_plan(self, positions):
        key = tuple((p._version, p.data_ptr()) for p in self.tensors.values())
        if self._plan is None or key != self._plan_key:
            self._build_plan()
            self._plan_key = key
        md, layers = self._plan[:2]
        if positions > self._rope_len:
            self._rope_len = round_up(positions, 1024)
            self._rope = {}
            for d, spec in zip(layers, self.config.layers):
                d.rope = self._rope_table(spec.mixer.rot_base, spec.mixer.rot_dims).data_ptr()
            md.rope_len = self._rope_len
        return md

    def _workspace(self, md, B, T, n_logits, keys):
        key = (B, T, n_logits, keys)
        ws = self._workspaces.get(key)
        if ws is None:
            nbytes = _lib.stack_lib().nc_stack_workspace_bytes(C.byref(md), B, T, n_logits, keys)
            held = sum(w.numel() for w in self._workspaces.values())
            if held + nbytes > self.WORKSPACE_CACHE_BYTES:
                self._workspaces.clear()
            ws = self._workspaces[key] = torch.empty(nbytes + 256, dtype=torch.uint8, device=self.get_device())
        off = (-ws.data_ptr()) % 256
        return ws.data_ptr() + off, ws.numel() - off

    # ---- forward
    @torch.no_grad()
    def _run(self, idx, kv_cache, rows=None, taps=False):
        """rows: None (all), or an int32 device tensor of flat indices batch_row * T + token.  Returns (logits, taps or None)."""
        if not idx.is_cuda:
            raise RuntimeError("the layer stack runs on the GPU only; there is no CPU fallback")
        assert idx.dtype == torch.long
        B, T = idx.shape
        if T > 1:
            # a prompt: worth one read-back to refuse ids outside the embedding table (a decode step is fed by the sampler)
            lo, hi = torch.aminmax(idx)
            if int(lo) < 0 or int(hi) >= self.config.vocab_size:
                raise IndexError(f"token id out of range: [{int(lo)}, {int(hi)}] for an embedding table of {self.config.vocab_size} rows")
        if kv_cache is None:
            kv_cache = self.new_cache(B, T)
        assert kv_cache.batch_size == B and kv_cache.dtype == self.dtype
        pos_max = kv_cache._pos_max
        assert pos_max + T <= kv_cache.max_seq_len, f"a cache of {kv_cache.max_seq_len} tokens cannot take {pos_max}+{T}"
        # (tables for the whole cache, so that they do not grow during a generation)
        md = self._ensure_plan(kv_cache.max_seq_len)
        lib = _lib.stack_lib()
        idx = idx.contiguous()
        n_logits = B * T if rows is None else rows.numel()
        logits = torch.empty(n_logits, self.config.vocab_size, dtype=torch.float32, device=idx.device)
        tap = torch.empty(len(self.run_list), B, T, self.width_p, dtype=torch.float32, device=idx.device) if taps else None
        cd = _lib.StackCacheDesc()
        cd.latents, cd.state_in, cd.state_out = kv_cache.pointers()
        cd.cache_seqlens = kv_cache.cache_seqlens.data_ptr()
        cd.batch, cd.max_seq_len, cd.pos_max = B, kv_cache.max_seq_len, pos_max
        cd.advance = T if rows is None else 0
        keys = kv_cache.max_seq_len if T == 1 else min(kv_cache.max_seq_len, round_up(pos_max + T, 256))
        ws_ptr, ws_bytes = self._workspace(md, B, T, n_logits, keys)
        rc = lib.nc_stack_forward(C.byref(md), C.byref(cd), idx.data_ptr(), B, T, rows.data_ptr() if rows is not None else None, n_logits,
                                  logits.data_ptr(), ws_ptr, ws_bytes, tap.data_ptr() if taps else None, torch.cuda.current_stream().cuda_stream)
        _lib.check(rc, lib)
        if cd.advance:
            kv_cache.note_advanced(T)
        else:
            kv_cache.advance(T)
        return logits, tap

    def forward(self, idx, targets=None, kv_cache=None, loss_reduction='mean'):
        """fp32 logits [B,T,vocab].  The cache is appended in place and advanced by T."""
        if targets is not None:
            raise NotImplementedError("training loss is outside the inference path implemented here")
        return self._run(idx, kv_cache)[0].view(*idx.shape, self.config.vocab_size)

    def forward_last(self, idx, kv_cache=None):
        """Logits of the last position of every row only, [B,vocab]: what Engine.generate consumes."""
        B, T = idx.shape
        if T == 1:
            return self._run(idx, kv_cache)[0]
        rows = torch.arange(T - 1, B * T, T, dtype=torch.int32, device=idx.device)
        return self._run(idx, kv_cache, rows)[0]

    def forward_at(self, idx, places, kv_cache=None):
        """Logits of the given flat places (batch row * T + token), [len(places), vocab]; the list may be empty."""
        assert all(0 <= p < idx.numel() for p in places)
        if list(places) == list(range(idx.numel())):
            return self._run(idx, kv_cache)[0]
        return self._run(idx, kv_cache, torch.tensor(list(places), dtype=torch.int32, device=idx.device))[0]

    def forward_tapped(self, idx, kv_cache=None):
        """(logits [B,T,vocab], residual stream after every layer run, fp32 [runs,B,T,n_embd]) for layer-by-layer comparisons."""
        logits, tap = self._run(idx, kv_cache, taps=True)
        return logits.view(*idx.shape, self.config.vocab_size), tap[..., :self.config.n_embd]
