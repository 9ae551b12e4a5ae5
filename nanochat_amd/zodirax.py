"""Zodirax: a small decoder whose layers, listed in its config.json, are a selective scan, or a window attention (kept first tokens, a sink
per head) beside a lightning attention (linear attention with a fixed decay per head); every sublayer reads the residual stream itself and
its output is normed; SwiGLU feed-forwards or none; the embedding table is the output matrix.

The design's config.json keys and tensor names are read here; the mechanisms are those of stack.py."""
from .stack import DenseSwiglu, LayerSpec, LayerStack, Retention, Rotation, SelectiveScan, SideBySide, StackConfig, WindowAttention

ARCHITECTURE = "Zodirax"


def _rotation(m):
    scaling = m.get("scaling") or {}
    return Rotation(base=float(m["base"]), dims=m["dims"], **{k: float(scaling[k]) for k in ("factor", "low", "high", "original") if scaling})


def _mixer(kind, m):
    if kind == "mamba1":
        return SelectiveScan(inner=m["inner"], state=m["state"], conv=m["conv"], dt_rank=m["dt_rank"])
    if kind == "parallel":
        a, r = m["left"], m["right"]
        left = WindowAttention(heads=a["heads"], kv_heads=a["kv_heads"], dim=a["dim"], vdim=a["vdim"], scale=float(a["scale"]), window=a["mask"]["size"],
                               keep_first=a["mask"]["keep_first"], rotation=_rotation(a["rot"]))
        right = Retention(heads=r["heads"], dim=r["dim"], vdim=r["vdim"], decay=[float(d) for d in r["decay"]], k_scale=1.0, silu_qkv=True, joint_norm=True)
        return SideBySide(left, right, float(m["left_scale"]), float(m["right_scale"]))
    raise ValueError(f"unknown mixer {kind!r}")


def _feed_forward(m):
    if m is None:
        return None
    if m["kind"] == "dense":
        return DenseSwiglu(ff=m["ff"])
    raise ValueError(f"unknown feed-forward {m['kind']!r}")


def stack_config(cfg):
    """StackConfig of a config.json dictionary."""
    return StackConfig(
        vocab_size=cfg["vocab"], n_embd=cfg["width"],
        layers=[LayerSpec(_mixer(layer["type"], layer["mixer"]), _feed_forward(layer.get("mlp"))) for layer in cfg["layers"]],
        eps=float(cfg["norm"]["eps"]), embed_scale=float(cfg["embedding"]["scale"]), block="post_norm", norm="rms", norm_offset=1.0, tied_head=True)


class Zodirax(LayerStack):
    stack_config = staticmethod(stack_config)
