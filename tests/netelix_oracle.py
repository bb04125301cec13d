"""A plain, slow restatement of the Netelix design in float64 on the CPU, one function per mechanism, written from the
design's equations (it shares no code with hydrainfer_amd).  Weights are a dict under the checkpoint's tensor names; the
configuration is the dict config.json holds.  Whole sequences only: no cache, no state slots, no batching — what the
engine must reproduce however it cuts and batches the work."""
from typing import Dict, List, Optional

import torch

F = torch.float64


def over_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x * (x.square().mean(-1, keepdim=True) + eps).rsqrt()


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


# ---------------------------------------------------------------------------------------------- rotations
def turned(x: torch.Tensor, positions: torch.Tensor, dims: int, base: float, neighbours: bool) -> torch.Tensor:
    """x [n, heads, dim] with its first `dims` channels turned by the token's position; partners are channels 2 i, 2 i + 1
    (neighbours) or i, i + dims / 2."""
    out = x.clone()
    for i in range(dims // 2):
        a, b = (2 * i, 2 * i + 1) if neighbours else (i, i + dims // 2)
        angle = positions.to(F) * base ** (-2.0 * i / dims)
        c, s = torch.cos(angle)[:, None], torch.sin(angle)[:, None]
        out[..., a] = x[..., a] * c - x[..., b] * s
        out[..., b] = x[..., b] * c + x[..., a] * s
    return out


# ---------------------------------------------------------------------------------------------- linear attention
def decayed_sum(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay: List[float], state: Optional[torch.Tensor] = None):
    """q, k [n, heads, dim], v [n, heads, vdim]: S <- decay_h S + k v^T, o = S^T q.  -> (o [n, heads, vdim], last S)."""
    n, H, D = q.shape
    d = torch.tensor(decay, dtype=F)[:, None, None]
    S = torch.zeros(H, D, v.shape[-1], dtype=F) if state is None else state.clone()
    o = torch.zeros(n, H, v.shape[-1], dtype=F)
    for t in range(n):
        S = d * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(1)
    return o, S


def retention(h, W, p, m, eps, shared=None):
    n, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q, k, v = (h @ W[p + s].T for s in "qkv")
    q, k, v = q.reshape(n, H, D), k.reshape(n, H, D), v.reshape(n, H, V)
    if m.get("rot"):
        pos = torch.arange(n)
        q, k = (turned(z, pos, m["rot"]["dims"], m["rot"]["base"], neighbours=False) for z in (q, k))
    o, _ = decayed_sum(q, k * D ** -0.5, v, m["decay"])
    return (over_rms(o, eps).reshape(n, H * V) * silu(h @ W[p + "g"].T)) @ W[p + "o"].T


def lightning(h, W, p, m, eps, shared=None):
    n, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q, k, v = (silu(h @ W[p + s].T) for s in "qkv")
    o, _ = decayed_sum(q.reshape(n, H, D), k.reshape(n, H, D), v.reshape(n, H, V), m["decay"])
    o = over_rms(o.reshape(n, H * V), eps) * W[p + "norm"]
    return (o * sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


# ---------------------------------------------------------------------------------------------- attention
def head_norm(x, w, eps):
    return over_rms(x, eps) * w


def mixed_values(v, first, lam):
    return (1.0 - lam) * v + lam * first


def attend(q, k, v, scale: float, window: Optional[int]) -> torch.Tensor:
    """q [n, H, dim] over k [n, G, dim], v [n, G, vdim] of the same sequence; query head h reads key head h // (H / G)."""
    n, H, G = q.shape[0], q.shape[1], k.shape[1]
    back = torch.arange(n)[:, None] - torch.arange(n)[None, :]
    seen = (back >= 0) & (back < (window if window else n + 1))
    o = torch.zeros(n, H, v.shape[-1], dtype=F)
    for h in range(H):
        g = h // (H // G)
        s = torch.where(seen, q[:, h] @ k[:, g].T * scale, torch.tensor(float("-inf"), dtype=F))
        o[:, h] = torch.softmax(s, -1) @ v[:, g]
    return o


def attention(h, W, p, m, eps, shared=None):
    """shared: a dict that carries the first value-mixing layer's values through the model."""
    n, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k = (h @ W[p + "q"].T).reshape(n, H, D), (h @ W[p + "k"].T).reshape(n, G, D)
    v = (h @ W[p + "v"].T).reshape(n, G, V)
    q, k = head_norm(q, W[p + "q.norm"], eps), head_norm(k, W[p + "k.norm"], eps)
    if m.get("rot"):
        pos = torch.arange(n)
        q, k = (turned(z, pos, m["rot"]["dims"], m["rot"]["base"], neighbours=True) for z in (q, k))
    if m.get("v_mix"):
        if "v" not in shared:
            shared["v"] = v
        else:
            v = mixed_values(v, shared["v"], W[p + "vmix"])
    o = attend(q, k, v, m["scale"], (m.get("mask") or {}).get("size"))
    return o.reshape(n, H * V) @ W[p + "o"].T


# ---------------------------------------------------------------------------------------------- feed-forward, model
def dense_ff(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


MIXERS = {"retention": retention, "lightning": lightning, "attention": attention}


def forward(cfg: dict, weights: Dict[str, torch.Tensor], tokens: List[int], layers_out: Optional[list] = None) -> torch.Tensor:
    """Logits [n, vocab] of one whole sequence; layers_out (a list) receives the residual after every layer."""
    W = {k: v.to(F) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    shared = {}
    x = over_rms(W["embed"][torch.tensor(tokens)], eps) * W["embed.norm"]
    for i, l in enumerate(cfg["layers"]):
        p = f"l{i}."
        y = MIXERS[l["type"]](x, W, p + "mix.", l["mixer"], eps, shared)
        x = x + over_rms(y, eps) * W[p + "norm1"] * W[p + "ls1"]
        if l.get("mlp") is not None:
            y = dense_ff(x, W, p + "mlp.")
            x = x + over_rms(y, eps) * W[p + "norm2"] * W[p + "ls2"]
        if layers_out is not None:
            layers_out.append(x.clone())
    return (over_rms(x, eps) * W["final.norm"]) @ W["head"].T


def greedy(cfg, weights, prompt: List[int], n_new: int):
    """(tokens generated greedily, top-1 margin of every step)."""
    toks, out, margins = list(prompt), [], []
    for _ in range(n_new):
        top = torch.topk(forward(cfg, weights, toks)[-1], 2)
        out.append(int(top.indices[0]))
        margins.append(float(top.values[0] - top.values[1]))
        toks.append(out[-1])
    return out, margins
