"""Plain restatement of the Palilix decoder (test infrastructure only): one function per mechanism, a Python loop wherever a loop is
the definition, no cache, no batching, no fusion.  Everything runs in the dtype of the weights it is given (float64 in the tests).

A model is (config dict, {tensor name: tensor}); a sequence is a list of token ids; every function works on one sequence [T, ...].

    x_0 = E[token] * s
    before pass t of the looped layers:  x <- x + (x_0 if t > 0) + step_t
    layer:   h = LN(x),  x <- x + mixer(h) + ff(h)
    logits = cap * tanh(head LN(x) * a / cap)
"""
import math

import torch


# ------------------------------------------------------------------------------------------------ norms, activations, rotation
def rms_norm(x, eps, weight=None):
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if weight is None else y * weight


def layer_norm(x, weight, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * weight


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def silu(z):
    return z * torch.sigmoid(z)


def clamped_glu(gate, up, limit):
    g, u = gate.clamp(max=limit), up.clamp(-limit, limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1)


def rotate(x, pos, base, dims):
    """x [..., D] at integer positions `pos` (broadcast over the leading axes of x but the last): the first `dims` entries turn in
    pairs (i, i + dims/2) by pos * base^(-2i/dims), the others pass."""
    half = dims // 2
    freq = torch.tensor([base ** (-2.0 * i / dims) for i in range(half)], dtype=torch.float64).to(x.dtype)
    a = pos.to(x.dtype).unsqueeze(-1) * freq
    c, s = a.cos(), a.sin()
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., dims:]], dim=-1)


# ------------------------------------------------------------------------------------------------ mixers
def latent_attention(h, w, cfg, eps, pos0=0):
    """h [T, width] -> [T, width].  Per head, over the keys j <= i: softmax((q_n . k_n + q_r . k_r) * scale) v, where k_n and v are
    linear in the normed latent and k_r is one rotated part for all heads."""
    T = h.shape[0]
    H, dn, dr, dv, r = cfg["heads"], cfg["dim"], cfg["rot_dim"], cfg["vdim"], cfg["kv_rank"]
    pos = torch.arange(pos0, pos0 + T)
    q = (h @ w["q"].T).view(T, H, dn + dr)
    q_n, q_r = q[..., :dn], rotate(q[..., dn:], pos[:, None], cfg["rot"]["base"], cfg["rot"]["dims"])
    dkv = h @ w["dkv"].T
    c = rms_norm(dkv[:, :r], eps, w["dkv.norm"])
    k_r = rotate(dkv[:, r:], pos, cfg["rot"]["base"], cfg["rot"]["dims"])
    k_n, v = (c @ w["uk"].T).view(T, H, dn), (c @ w["uv"].T).view(T, H, dv)
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for i in range(T):
        for head in range(H):
            s = (k_n[:i + 1, head] @ q_n[i, head] + k_r[:i + 1] @ q_r[i, head]) * cfg["scale"]
            out[i, head] = torch.softmax(s, dim=0) @ v[:i + 1, head]
    return out.reshape(T, H * dv) @ w["o"].T


def retention(h, w, cfg, eps, pos0=0, state=None):
    """h [T, width] -> ([T, width], state [H, dim, vdim]).  S <- decay S + k v^T, o = S^T q, token by token."""
    T = h.shape[0]
    H, dk, dv = cfg["heads"], cfg["dim"], cfg["vdim"]
    pos = torch.arange(pos0, pos0 + T)[:, None]
    q = rotate((h @ w["q"].T).view(T, H, dk), pos, cfg["rot"]["base"], cfg["rot"]["dims"])
    k = rotate((h @ w["k"].T).view(T, H, dk), pos, cfg["rot"]["base"], cfg["rot"]["dims"]) * dk ** -0.5
    v = (h @ w["v"].T).view(T, H, dv)
    decay = torch.tensor(cfg["decay"], dtype=h.dtype)[:, None, None]
    S = torch.zeros(H, dk, dv, dtype=h.dtype) if state is None else state
    o = torch.zeros(T, H, dv, dtype=h.dtype)
    for t in range(T):
        S = decay * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(1)
    o = rms_norm(o, eps).reshape(T, H * dv)
    return (o * silu(h @ w["g"].T)) @ w["o"].T, S


# ------------------------------------------------------------------------------------------------ feed-forward
def dense_ff(h, w):
    return gelu_tanh(h @ w["up"].T) @ w["down"].T


def expert(h, gate, up, down, limit):
    return clamped_glu(h @ gate.T, h @ up.T, limit) @ down.T


def route(h, router, top):
    """(indices [T, top], weights [T, top]): softmax over all experts, the largest `top`, their scores over their own sum."""
    s = torch.softmax(h @ router.T, dim=-1)
    val, idx = s.topk(top, dim=-1)
    return idx, val / (val.sum(-1, keepdim=True) + 1e-20)


def moe(h, w, cfg):
    idx, wt = route(h, w["router"], cfg["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(idx[t].tolist(), wt[t]):
            out[t] += a * expert(h[t], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"], cfg["expert"]["limit"])
    if cfg.get("shared"):
        out = out + expert(h, w["shared.gate"], w["shared.up"], w["shared.down"], cfg["shared"]["limit"])
    return out


def feed_forward(h, w, cfg):
    return dense_ff(h, w) if cfg["kind"] == "dense" else moe(h, w, cfg)


# ------------------------------------------------------------------------------------------------ the model
def sub(weights, prefix):
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def layer_runs(cfg):
    """[(layer, pass or None)] in the order they run; pass is the loop's pass number for the first layer of each pass only."""
    n = len(cfg["layers"])
    loop = cfg.get("loop") or {"start": 0, "stop": 0, "times": 1}
    runs = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        runs += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return runs + [(i, None) for i in range(loop["stop"], n)]


def forward(cfg, weights, tokens, taps=None):
    """Logits [T, vocab] of one sequence; `taps`, a list, receives the residual stream after every layer run."""
    eps = cfg["norm"]["eps"]
    x0 = weights["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
    x = x0
    for i, t in layer_runs(cfg):
        if t is not None:
            if t > 0:
                x = x + x0
            x = x + weights["loop.step"][t]
        lc = cfg["layers"][i]
        h = layer_norm(x, weights[f"l{i}.norm1"], eps)
        mix = sub(weights, f"l{i}.mix.")
        y = latent_attention(h, mix, lc["mixer"], eps) if lc["type"] == "latent_attention" else retention(h, mix, lc["mixer"], eps)[0]
        if lc["mlp"]:
            y = y + feed_forward(h, sub(weights, f"l{i}.mlp."), lc["mlp"])
        x = x + y
        if taps is not None:
            taps.append(x)
    logits = (layer_norm(x, weights["final.norm"], eps) @ weights["head"].T) * cfg["logit_scale"]
    cap = cfg.get("logit_softcap")
    return cap * torch.tanh(logits / cap) if cap else logits
