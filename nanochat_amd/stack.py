"""Decoders made of configured layers: any order of mixers and feed-forwards, a run of layers that may repeat with the same weights.

A layer is `x += mixer(h) + ff(h)` with `h = norm(x)` (block "parallel"), or `x += norm1(mixer(x)); x += norm2(ff(x))` (block
"post_norm").  The mechanisms are classes of their own with their sizes and constants as fields; each knows the tensors it needs, how they
are packed for the kernels and what it keeps per sequence:

    mixers         LatentAttention, Retention, WindowAttention, SelectiveScan, SideBySide (two of them on the same input)
    feed-forwards  DenseGelu, DenseSwiglu, Experts (clamped GLU experts, softmax router, optional shared expert)

`LayerStack` is the model: weights by name, a packed plan that is rebuilt whenever a weight changes, and a forward that is one native
call (nc_stack_forward).  It has the surface the Engine and the harness use on every model of this package (forward, forward_last,
new_cache, get_device, the cost accounting).  A design is a class that turns its configuration into a StackConfig (palilix.py,
zodirax.py).

Two storage types: bfloat16 (matrix products in bf16 with 32-bit sums; residual stream, norms, angles, scores, router and recurrent
state in 32-bit), and float32 (everything in true 32-bit).
"""
import ctypes as C
import math
from dataclasses import dataclass, field

import torch
import torch.nn as nn

from . import _lib, ops
from .checkpoint import read_config, read_safetensors

PAD = ops.STACK_PAD
WEIGHT_FIELDS = ("w_uk_t", "w_ukv", "w_x", "w_dt", "w_dt_t")       # of a mixer's descriptor: in the storage type; the others are fp32


def round_up(n, m):
    return -(-n // m) * m


def padded(t, *shape):
    """t in the leading corner of a zero tensor of `shape`."""
    out = torch.zeros(shape, dtype=t.dtype, device=t.device)
    out[tuple(slice(0, n) for n in t.shape)] = t
    return out


@dataclass(frozen=True)
class Rotation:
    """Rotary positions: pair i of `dims` leading dimensions turns by position * base^(-2i/dims).  With `factor`, wavelengths longer than
    original / low are stretched by it, those shorter than original / high are kept, and a ramp in 1 / wavelength joins the two."""
    base: float
    dims: int
    factor: float = 1.0
    low: float = 1.0
    high: float = 1.0
    original: float = 0.0           # 0: no stretching

    def frequencies(self):
        i = torch.arange(self.dims // 2, dtype=torch.float64)
        f = self.base ** (-2.0 * i / max(self.dims, 1))
        if not self.original:
            return f
        turns = self.original * f / (2 * math.pi)             # original / wavelength
        if self.high == self.low:
            keep = (turns > self.high).double()
        else:
            keep = ((turns - self.low) / (self.high - self.low)).clamp(0.0, 1.0)
        return (1 - keep) * f / self.factor + keep * f


NO_ROTATION = Rotation(1.0, 0)
ROW_CACHE, STATE_CACHE = 0, 1       # what a mixer keeps: a row per token, or a state per sequence


class Mixer:
    """What the layers ask of a mixer.  `cols` rows of the input matrix are its projections, `out` columns of the output matrix take its
    result; `row_width` values per token or a state of `state_shape` are kept per sequence.  Tensors named in `fp32` stay 32-bit."""
    cache = ROW_CACHE
    row_width = 0
    state_shape = ()
    rotation = NO_ROTATION
    out_scale = 1.0
    fp32 = ()
    per_key = ()                    # tensors applied per key or query, counted in flops() rather than as weights a token passes
    scales_output = False

    def prefill_flops(self, tokens):
        return sum(self.flops(n) for n in range(1, tokens + 1))

    @property
    def parts(self):
        """[(prefix of its tensors' names, mixer)]: itself, or what it is made of."""
        return [("", self)]


# ------------------------------------------------------------------------------------------------ mixers
@dataclass
class LatentAttention(Mixer):
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
    per_key = ("uk", "uv")

    def __post_init__(self):
        assert self.rot_dim % 2 == 0, f"rotated part of odd size {self.rot_dim}"
        self.rotation = Rotation(self.rot_base, self.rot_dim)
        self.dim_p, self.rot_p, self.rank_p = round_up(self.dim, 32), round_up(self.rot_dim, 32), round_up(self.rank, PAD)
        # the heads' values side by side fill whole K-steps of the output matrix
        self.vdim_p = round_up(self.vdim, 16 * (4 // math.gcd(self.heads, 4)))
        self.cols = self.heads * (self.dim_p + self.rot_p) + self.rank_p + self.rot_p
        self.out = self.heads * self.vdim_p
        self.row_width = self.rank_p + self.rot_p

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
        d.heads, d.dim, d.dim_p, d.vdim, d.vdim_p, d.rot_dim, d.rot_p = self.heads, self.dim, self.dim_p, self.vdim, self.vdim_p, self.rot_dim, self.rot_p
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
class Retention(Mixer):
    """Linear attention with one fixed decay per head, rotary positions on the first `rot_dims` dimensions of q and k.  `decay` holds one
    factor per head.  q, k and v pass silu if `silu_qkv`.  The outputs are normed per head and multiplied by silu(gate), or (`joint_norm`)
    normed over all heads at once with a weight and multiplied by sigmoid(gate)."""
    heads: int
    dim: int
    vdim: int
    decay: list
    rot_dims: int = 0
    rot_base: float = 1.0
    k_scale: float = field(default=None)
    silu_qkv: bool = False
    joint_norm: bool = False

    kind = 1
    cache = STATE_CACHE

    def __post_init__(self):
        assert len(self.decay) == self.heads, f"{len(self.decay)} decays for {self.heads} heads"
        assert self.rot_dims % 2 == 0 and self.rot_dims <= self.dim
        self.rotation = Rotation(self.rot_base, self.rot_dims)
        self.scales_output = self.joint_norm
        if self.k_scale is None:
            self.k_scale = self.dim ** -0.5
        # sizes the kernels hold a state in registers for; larger ones go through memory
        sizes = [n for n in (64, 128, 256)]
        self.dim_p = next((n for n in sizes if n >= self.dim), round_up(self.dim, PAD))
        self.vdim_p = next((n for n in sizes if n >= max(self.vdim, 128 if self.dim_p == 256 else 0)), round_up(self.vdim, PAD))
        self.cols = 2 * self.heads * (self.dim_p + self.vdim_p)
        self.out = self.heads * self.vdim_p
        self.state_shape = (self.heads, self.dim_p, self.vdim_p)

    def tensors(self, width):
        H = self.heads
        return {"q": (H * self.dim, width), "k": (H * self.dim, width), "v": (H * self.vdim, width), "g": (H * self.vdim, width),
                "o": (width, H * self.vdim)} | ({"norm": (H * self.vdim,)} if self.joint_norm else {})

    def pack(self, w):
        H, width = self.heads, w["q"].shape[1]

        def heads(t, n, n_p):
            return padded(t.view(H, n, width), H, n_p, width).view(H * n_p, width)
        rows = [heads(w["q"], self.dim, self.dim_p), heads(w["k"], self.dim, self.dim_p), heads(w["v"], self.vdim, self.vdim_p),
                heads(w["g"], self.vdim, self.vdim_p)]
        o = padded(w["o"].view(width, H, self.vdim), width, H, self.vdim_p).view(width, H * self.vdim_p)
        decay = torch.tensor(self.decay, dtype=torch.float32)
        log2 = torch.log2(decay.double()).clamp(min=-1000.0).float()          # a decay of 0 forgets everything: 2^-1000 is 0 as well
        extra = {"decay": torch.stack([decay, log2], dim=1).to(o.device)}
        if self.joint_norm:
            extra["out_norm_w"] = padded(w["norm"].float().view(H, self.vdim), H, self.vdim_p)
        return torch.cat(rows), o, extra

    def describe(self, d):
        d.heads, d.dim, d.dim_p, d.vdim, d.vdim_p, d.score_scale = self.heads, self.dim, self.dim_p, self.vdim, self.vdim_p, self.k_scale
        d.silu_qkv, d.gate = int(self.silu_qkv), int(self.joint_norm)

    def flops(self, keys):
        return 4 * self.heads * self.dim * self.vdim

    def prefill_flops(self, tokens):
        return tokens * self.flops(0)

    def read_elements(self, keys):
        return 0, 2 * self.heads * self.dim * self.vdim


@dataclass
class WindowAttention(Mixer):
    """Grouped-query softmax attention over the last `window` keys and, however far away, the first `keep_first`.  q, k and v have biases;
    q and k are RMS-normed over all heads at once, then turned; a number per head (the sink) counts in the softmax's denominator."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int
    keep_first: int
    rotation: Rotation = NO_ROTATION
    out_scale: float = 1.0

    kind = 2
    scales_output = True

    def __post_init__(self):
        assert self.kv_heads >= 1 and self.heads % self.kv_heads == 0, f"{self.heads} query heads on {self.kv_heads} key heads"
        assert self.rotation.dims % 2 == 0 and self.rotation.dims <= self.dim, f"{self.rotation.dims} of {self.dim} dimensions turn"
        assert self.window >= 1 and self.keep_first >= 0
        self.dim_p = round_up(self.dim, 32)
        self.vdim_p = round_up(self.vdim, 16 * (4 // math.gcd(self.heads, 4)))
        self.cols = (self.heads + self.kv_heads) * self.dim_p + self.kv_heads * self.vdim_p
        self.out = self.heads * self.vdim_p
        self.row_width = self.kv_heads * (self.dim_p + self.vdim_p)

    def tensors(self, width):
        out = {"o": (width, self.heads * self.vdim), "sink": (self.heads,), "q.norm": (self.heads * self.dim,), "k.norm": (self.kv_heads * self.dim,)}
        for name, n in (("q", self.heads * self.dim), ("k", self.kv_heads * self.dim), ("v", self.kv_heads * self.vdim)):
            out |= {name: (n, width), f"{name}.b": (n,)}
        return out

    def pack(self, w):
        H, G, width = self.heads, self.kv_heads, w["q"].shape[1]
        sizes = {"q": (H, self.dim, self.dim_p), "k": (G, self.dim, self.dim_p), "v": (G, self.vdim, self.vdim_p)}
        rows = [padded(w[name].view(n, d, width), n, d_p, width).view(n * d_p, width) for name, (n, d, d_p) in sizes.items()]
        bias = [padded(w[f"{name}.b"].float().view(n, d), n, d_p).view(-1) for name, (n, d, d_p) in sizes.items()]
        norms = {f"{name}_norm_w": padded(w[f"{name}.norm"].float().view(n, d), n, d_p) for name, (n, d, d_p) in sizes.items() if name != "v"}
        o = padded(w["o"].view(width, H, self.vdim), width, H, self.vdim_p).view(width, H * self.vdim_p)
        return torch.cat(rows), o, {"qkv_bias": torch.cat(bias), "sink": w["sink"].float(), **norms}

    def describe(self, d):
        d.heads, d.kv_heads, d.dim, d.dim_p, d.vdim, d.vdim_p = self.heads, self.kv_heads, self.dim, self.dim_p, self.vdim, self.vdim_p
        d.score_scale, d.window, d.keep_first = self.scale, min(self.window, 1 << 30), min(self.keep_first, 1 << 30)

    def seen(self, keys):
        return min(keys, self.window + self.keep_first)

    def flops(self, keys):
        return 2 * self.heads * self.seen(keys) * (self.dim + self.vdim)

    def read_elements(self, keys):
        return self.seen(keys) * self.kv_heads * (self.dim + self.vdim), 0


@dataclass
class SelectiveScan(Mixer):
    """A causal convolution of `conv` taps per channel, then `state` linear recurrences per channel whose step sizes, inputs and read-outs
    come from the token; gated by silu of a second projection."""
    inner: int
    state: int
    conv: int
    dt_rank: int

    kind = 3
    cache = STATE_CACHE
    fp32 = ("conv", "A_log")
    scales_output = True

    def __post_init__(self):
        assert min(self.inner, self.state, self.conv, self.dt_rank) >= 1
        assert self.state <= 256, f"{self.state} states per channel"
        self.inner_p, self.dt_rank_p = round_up(self.inner, PAD), round_up(self.dt_rank, PAD)
        # 4, 8, 12 or 16 states in each of 1, 2, 4, 8 or 16 lanes
        self.state_p = min(n << k for n in (4, 8, 12, 16) for k in range(5) if n << k >= self.state)
        self.bc_p = round_up(self.state_p, 16)
        self.cols, self.out = 2 * self.inner_p, self.inner_p
        self.state_shape = (self.state_p + self.conv - 1, self.inner_p)

    def tensors(self, width):
        n = self.inner
        return {"in": (2 * n, width), "conv": (n, self.conv), "conv.b": (n,), "x": (self.dt_rank + 2 * self.state, n), "dt": (n, self.dt_rank), "dt.b": (n,),
                "A_log": (n, self.state), "D": (n,), "o": (width, n)}

    def pack(self, w):
        n, n_p, width = self.inner, self.inner_p, w["in"].shape[1]
        rows = padded(w["in"].view(2, n, width), 2, n_p, width).view(2 * n_p, width)
        step, B, C = w["x"].split([self.dt_rank, self.state, self.state])
        w_x = torch.cat([padded(step, self.dt_rank_p, n_p), padded(B, self.bc_p, n_p), padded(C, self.bc_p, n_p)])
        w_dt = padded(w["dt"], n_p, self.dt_rank_p)
        a = -torch.exp(w["A_log"].double()) * math.log2(math.e)
        return rows, padded(w["o"], width, n_p), {
            "conv_w": padded(w["conv"].float().T, self.conv, n_p), "conv_b": padded(w["conv.b"].float(), n_p), "w_x": w_x, "w_dt": w_dt, "w_dt_t": w_dt.T,
            "dt_b": padded(w["dt.b"].float(), n_p), "a_log2": padded(a.T, self.state_p, n_p).float(), "skip": padded(w["D"].float(), n_p)}

    def describe(self, d):
        d.inner, d.inner_p, d.state, d.state_p, d.taps = self.inner, self.inner_p, self.state, self.state_p, self.conv
        d.dt_rank, d.dt_rank_p = self.dt_rank, self.dt_rank_p

    def flops(self, keys):
        return 6 * self.inner * self.state

    def prefill_flops(self, tokens):
        return tokens * self.flops(0)

    def read_elements(self, keys):
        return 0, 2 * self.inner * (self.state + self.conv - 1)


@dataclass
class SideBySide:
    """Two mixers on the same input; the layer's mixer result is the sum of theirs, each times its scale."""
    left: Mixer
    right: Mixer
    left_scale: float = 1.0
    right_scale: float = 1.0

    def __post_init__(self):
        for mixer, scale in ((self.left, self.left_scale), (self.right, self.right_scale)):
            assert scale == 1.0 or mixer.scales_output, f"{type(mixer).__name__} does not scale its result"
            mixer.out_scale = scale

    @property
    def parts(self):
        return [("left.", self.left), ("right.", self.right)]

    def tensors(self, width):
        return {prefix + k: s for prefix, m in self.parts for k, s in m.tensors(width).items()}


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
class DenseSwiglu:
    """down (silu(gate h) * (up h))."""
    ff: int

    kind = 3

    def __post_init__(self):
        self.ff_p = round_up(self.ff, PAD)
        self.router_cols, self.ff_cols = 0, 2 * self.ff_p

    def tensors(self, width):
        return {"gate": (self.ff, width), "up": (self.ff, width), "down": (width, self.ff)}

    def pack(self, w, width_p):
        return None, interleaved(w["gate"], w["up"], self.ff_p, width_p), padded(w["down"], width_p, self.ff_p), {}

    def describe(self, d):
        d.ff_limit = 0.0

    def active_params(self, width):
        return 3 * self.ff * width


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
    mixer: object                   # a Mixer, or two SideBySide
    ff: object = None               # None: no feed-forward

    @property
    def mixers(self):
        return [m for _, m in self.mixer.parts]


BLOCKS = {"parallel": 0, "post_norm": 1}
NORMS = {"layer": 0, "rms": 1}


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
    block: str = "parallel"         # "parallel": one norm, both sublayers read it; "post_norm": one after the other, a norm on each output
    norm: str = "layer"             # "layer" or "rms"
    norm_offset: float = 0.0        # added to the stored weights of the model's norms (1: stored around zero)
    tied_head: bool = False         # the output matrix is the embedding table
    sequence_len: int = 2048        # how far a generation without a token limit goes; the model itself has no limit

    def __post_init__(self):
        if self.block not in BLOCKS or self.norm not in NORMS:
            raise ValueError(f"block {self.block!r}, norm {self.norm!r}")
        if self.block == "post_norm" and (self.norm != "rms" or any(isinstance(layer.ff, Experts) for layer in self.layers)):
            raise ValueError("a post-norm block has RMS norms and dense feed-forwards")

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

    @classmethod
    def from_config(cls, cfg, dtype=torch.bfloat16):
        """A design's model (its class has a stack_config) from a config.json dictionary."""
        return cls(cls.stack_config(cfg), dtype)

    @classmethod
    def load(cls, model_dir, dtype=torch.bfloat16, device="cuda"):
        """The model in a folder with config.json and model.safetensors."""
        with torch.device("meta"):
            model = cls.from_config(read_config(model_dir), dtype)
        return model.load_tensors(read_safetensors(model_dir), torch.device(device)).eval()

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
                out |= {f"l{i}.norm2": (W,)} if config.block == "post_norm" else {}
                out |= {f"l{i}.mlp.{k}": s for k, s in layer.ff.tensors(W).items()}
        return out | {"final.norm": (W,)} | ({} if config.tied_head else {"head": (config.vocab_size, W)})

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
        """Take the weights by name, in the dtype they come in; names and shapes must be exactly the model's (the norm of a feed-forward
        that a layer does not have may be there)."""
        want = self.tensor_shapes(self.config)
        idle = {f"l{i}.norm2" for i, layer in enumerate(self.config.layers) if layer.ff is None and self.config.block == "post_norm"}
        missing, extra = sorted(set(want) - set(tensors)), sorted(set(tensors) - set(want) - idle)
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
        """(share_prompt_reads: every model's new_cache takes it; cached rows are read per sequence here)"""
        from .engine import StackCache
        mixers = self.run_mixers()
        return StackCache([m.row_width for m in mixers if m.cache == ROW_CACHE], [m.state_shape for m in mixers if m.cache == STATE_CACHE],
                          self.dtype, batch_size, seq_len, self.get_device(), prefill_from=prefill_from)

    def run_mixers(self):
        """The mixers in the order they run, a repeated layer's once per run."""
        return [m for i, _, _ in self.run_list for m in self.config.layers[i].mixers]

    # ---- cost accounting
    def num_active_matmul_params(self):
        """Weights a token is multiplied with, over all layer runs and the output matrix."""
        W, total = self.config.n_embd, self.config.vocab_size * self.config.n_embd
        for i, _, _ in self.run_list:
            layer = self.config.layers[i]
            for m in layer.mixers:
                total += sum(math.prod(s) for k, s in m.tensors(W).items() if len(s) == 2 and k not in m.per_key + m.fp32)
            total += layer.ff.active_params(W) if layer.ff is not None else 0
        return total

    def estimate_decode_flops(self, context_len):
        return 2 * self.num_active_matmul_params() + sum(m.flops(context_len) for m in self.run_mixers())

    def estimate_prefill_flops(self, num_tokens):
        return 2 * self.num_active_matmul_params() * num_tokens + sum(m.prefill_flops(num_tokens) for m in self.run_mixers())

    def kv_bytes_per_token(self):
        """Cache bytes that grow with the sequence (a recurrent state does not)."""
        es = self.dtype.itemsize
        return sum(m.read_elements(1)[0] for m in self.run_mixers()) * es

    def kv_read_bytes(self, context_len):
        """Cache bytes one decode step reads or writes per row."""
        parts = [m.read_elements(context_len) for m in self.run_mixers()]
        return sum(p[0] for p in parts) * self.dtype.itemsize + sum(p[1] for p in parts) * 4

    def streamed_weight_bytes(self):
        """Weight bytes one single-row decode step reads."""
        per_head = sum(math.prod(s) for m in self.run_mixers() for k, s in m.tensors(self.config.n_embd).items() if k in m.per_key)
        return (self.num_active_matmul_params() + per_head) * self.dtype.itemsize

    def describe(self):
        kinds = [" + ".join(type(m).__name__ for m in layer.mixers) for layer in self.config.layers]
        mix = ", ".join(f"{kinds.count(k)} {k}" for k in dict.fromkeys(kinds))
        return f"layers {len(kinds)} ({mix}), {len(self.run_list)} layer runs, dim {self.config.n_embd}"

    # ---- plan
    def _rope_table(self, rotation):
        """cos, sin of position * frequency, fp32 [len, dims/2, 2] (worked out in fp64: an angle of thousands of radians keeps its
        fraction)."""
        t = self._rope.get(rotation)
        if t is None:
            dev = self.get_device()
            ang = torch.outer(torch.arange(self._rope_len, dtype=torch.float64, device=dev), rotation.frequencies().to(dev))
            t = self._rope[rotation] = torch.stack([ang.cos(), ang.sin()], dim=-1).float().contiguous()
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

        def norm_weight(name):
            return own(padded(w[name].float() + cfg.norm_offset, Wp), torch.float32)

        def pick(prefix, fp32=()):
            mine = {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}
            return {k: v.to(self.dtype) if v.dim() > 1 and k not in fp32 else v for k, v in mine.items()}

        layers = (_lib.StackLayer * cfg.n_layer)()
        for i, spec in enumerate(cfg.layers):
            d, ff = layers[i], spec.ff
            rows, cols, extra = [], [], {}
            d.block, d.n_mixers = BLOCKS[cfg.block], len(spec.mixers)
            assert d.n_mixers <= _lib.STACK_MAX_MIXERS
            for j, (prefix, mixer) in enumerate(spec.mixer.parts):
                mix = d.mix[j]
                r, c, more = mixer.pack(pick(f"l{i}.mix.{prefix}", mixer.fp32))
                rows.append(padded(r, r.shape[0], Wp))
                cols.append(padded(c, Wp, mixer.out))
                mix.kind, mix.cols, mix.out, mix.out_scale, mix.rot_dims = mixer.kind, mixer.cols, mixer.out, mixer.out_scale, mixer.rotation.dims
                mixer.describe(mix)
                for name, t in more.items():
                    setattr(mix, name, own(t, self.dtype if name in WEIGHT_FIELDS else torch.float32))
                d.mix_cols += mixer.cols
                d.mix_out += mixer.out
            if ff is not None:
                router, first, last, extra = ff.pack(pick(f"l{i}.mlp."), Wp)
                d.ff, d.router_cols, d.ff_cols, d.ff_p = ff.kind, ff.router_cols, ff.ff_cols, ff.ff_p
                ff.describe(d)
                if cfg.block == "post_norm":
                    d.w_ff_in, d.w_ff_out, d.norm2_w = own(first, self.dtype), own(last, self.dtype), norm_weight(f"l{i}.norm2")
                else:
                    rows += [t for t in (router, first) if t is not None]
                    cols += [t for t in (last,) if t is not None]
            d.n_in, d.k_out = sum(t.shape[0] for t in rows), sum(t.shape[1] for t in cols)
            d.w_in, d.w_out = own(torch.cat(rows), self.dtype), own(torch.cat(cols, dim=1), self.dtype)
            d.norm_w = norm_weight(f"l{i}.norm1")
            for name, t in extra.items():
                setattr(d, name, own(t, self.dtype))
        runs = (_lib.StackRun * len(self.run_list))()
        used = {ROW_CACHE: 0, STATE_CACHE: 0}
        for r, (i, again, step) in zip(runs, self.run_list):
            r.layer, r.add_embedding, r.step = i, int(again), step
            for j, mixer in enumerate(cfg.layers[i].mixers):
                r.slot[j] = used[mixer.cache]
                used[mixer.cache] += 1
        md = _lib.StackModel()
        md.dtype, md.width, md.width_p, md.vocab = ops.STACK_DTYPES[self.dtype], cfg.n_embd, Wp, cfg.vocab_size
        md.n_layers, md.n_runs, md.max_k_out = cfg.n_layer, len(self.run_list), max(d.k_out for d in layers)
        md.norm = NORMS[cfg.norm]
        md.eps, md.embed_scale, md.logit_scale, md.logit_softcap = cfg.eps, cfg.embed_scale, cfg.logit_scale, cfg.logit_softcap
        md.embed = own(padded(w["embed"], cfg.vocab_size, Wp), self.dtype)
        md.head = md.embed if cfg.tied_head else own(padded(w["head"], cfg.vocab_size, Wp), self.dtype)
        md.final_norm_w = norm_weight("final.norm")
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
                for mix, mixer in zip(d.mix, spec.mixers):
                    mix.rope = self._rope_table(mixer.rotation).data_ptr() if mixer.rotation.dims else None
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
        cd.rows, cd.state_in, cd.state_out = kv_cache.pointers()
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
