"""Palilix: a small decoder whose layers, listed in its config.json, are latent attention or retention beside a dense or an expert
feed-forward (both sublayers read one layer norm), with a run of layers that repeats with the same weights.

The design's config.json keys and tensor names are read here; the mechanisms are those of stack.py."""
from .stack import DenseGelu, Experts, LatentAttention, LayerSpec, LayerStack, Retention, StackConfig

ARCHITECTURE = "Palilix"


def _mixer(kind, m):
    if kind == "latent_attention":
        if m["rot"]["dims"] != m["rot_dim"]:
            raise ValueError(f"the rotated part has {m['rot_dim']} dimensions, rot.dims is {m['rot']['dims']}")
        return LatentAttention(heads=m["heads"], dim=m["dim"], rot_dim=m["rot_dim"], vdim=m["vdim"], rank=m["kv_rank"], scale=float(m["scale"]),
                               rot_base=float(m["rot"]["base"]))
    if kind == "retention":
        return Retention(heads=m["heads"], dim=m["dim"], vdim=m["vdim"], decay=[float(d) for d in m["decay"]], rot_dims=m["rot"]["dims"],
                         rot_base=float(m["rot"]["base"]))
    raise ValueError(f"unknown mixer {kind!r}")


def _feed_forward(m):
    if m is None:
        return None
    if m["kind"] == "dense":
        return DenseGelu(ff=m["ff"])
    if m["kind"] == "moe":
        shared = m.get("shared") or {"ff": 0, "limit": 0.0}
        return Experts(experts=m["router"]["experts"], top=m["router"]["top"], ff=m["expert"]["ff"], limit=float(m["expert"]["limit"]),
                       shared_ff=shared["ff"], shared_limit=float(shared["limit"]))
    raise ValueError(f"unknown feed-forward {m['kind']!r}")


def stack_config(cfg):
    """StackConfig of a config.json dictionary."""
    loop = cfg.get("loop")
    return StackConfig(
        vocab_size=cfg["vocab"], n_embd=cfg["width"],
        layers=[LayerSpec(_mixer(layer["type"], layer["mixer"]), _feed_forward(layer.get("mlp"))) for layer in cfg["layers"]],
        eps=float(cfg["norm"]["eps"]), embed_scale=float(cfg["embedding"]["scale"]), logit_scale=float(cfg["logit_scale"]),
        logit_softcap=float(cfg.get("logit_softcap") or 0.0),
        **(dict(loop_start=loop["start"], loop_stop=loop["stop"], loop_times=loop["times"], loop_steps=True) if loop else {}))


class Palilix(LayerStack):
    stack_config = staticmethod(stack_config)
