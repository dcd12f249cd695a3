"""A plain, slow Zokunex: whole sequences, no cache, one function for each mechanism.

Zokunex is a decoder-only model whose layers are listed in its configuration. The sub-layers read the residual stream
itself, and a layer norm (weight, no bias) stands behind each of them: ``x += norm1(mixer(x)); x += norm2(ff(x))``.
A mixer is one of two:

* ``mlstm``: a matrix memory per head with an exponential input gate and a sigmoid forget gate, both softly capped,
  kept in range by a running maximum; the readout is divided by a normaliser that is a memory of its own;
* ``latent_attention``: keys and values of all heads expanded from one latent row per token, one rotated key part
  (half-split pairs) that the heads share, softmax over every earlier key, a sigmoid gate per head.

The feed-forward squares the rectified hidden values, or is a mixture of small experts (exact GELU) chosen by their
softmax score plus a correction and weighed by the score alone; some experts are the identity. The logits are scaled.
This file shares no code with the engine: it parses config.json itself and reads the checkpoint with the
``safetensors`` package. Everything is float64.

Notation: T tokens, D width, H heads; ``h`` is a sub-layer's input [T, D]; weights are stored [out, in] and applied
as ``h @ W.T``.
"""
from __future__ import annotations

import json
import math
import os
from typing import Dict, List

import torch
from safetensors import safe_open


def read_model(model_dir: str, dtype=torch.float64):
    with open(os.path.join(model_dir, "config.json")) as f:
        cfg = json.load(f)
    w: Dict[str, torch.Tensor] = {}
    with safe_open(os.path.join(model_dir, "model.safetensors"), framework="pt") as f:
        for name in f.keys():
            w[name] = f.get_tensor(name).to(dtype)
    return cfg, w


# -- single mechanisms -------------------------------------------------------------------------------
def layer_norm(x, weight, eps):
    mean = x.mean(-1, keepdim=True)
    c = x - mean
    return c / torch.sqrt((c * c).mean(-1, keepdim=True) + eps) * weight


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def soft_cap(z, cap):
    return cap * torch.tanh(z / cap)


def log_sigmoid(z):
    return torch.minimum(z, torch.zeros_like(z)) - torch.log1p(torch.exp(-z.abs()))


def mlstm_gates(h, w, pre, cap):
    """Log input gate and log forget gate, [T, H] each."""
    i = soft_cap(h @ w[pre + "i"].T + w[pre + "i.b"], cap)
    f = log_sigmoid(soft_cap(h @ w[pre + "f"].T + w[pre + "f.b"], cap))
    return i, f


def matrix_memory(q, k, v, i, f):
    """One head, token by token: q, k [T, d], v [T, e], log gates i, f [T] -> [T, e]. The memory S and its normaliser
    n start at zero, the running maximum m at 0; S and n are the true memories times exp(-m)."""
    T, d = q.shape
    e = v.shape[1]
    S = torch.zeros(d, e, dtype=q.dtype)
    n = torch.zeros(d, dtype=q.dtype)
    m = torch.zeros((), dtype=q.dtype)
    out = torch.zeros(T, e, dtype=q.dtype)
    for t in range(T):
        m_new = torch.maximum(f[t] + m, i[t])
        keep, take = torch.exp(f[t] + m - m_new), torch.exp(i[t] - m_new)
        S = keep * S + take * torch.outer(k[t], v[t])
        n = keep * n + take * k[t]
        m = m_new
        out[t] = (S.T @ q[t]) / (torch.maximum((n @ q[t]).abs(), torch.exp(-m)) + 1e-6)
    return out


def mlstm_mixer(h, w, pre, m, eps):
    T = h.shape[0]
    H, d, e = m["heads"], m["dim"], m.get("vdim", m["dim"])
    q = (h @ w[pre + "q"].T).view(T, H, d) * d ** -0.5
    k = (h @ w[pre + "k"].T).view(T, H, d)
    v = (h @ w[pre + "v"].T).view(T, H, e)
    i, f = mlstm_gates(h, w, pre, m["gate_cap"])
    o = torch.stack([matrix_memory(q[:, a], k[:, a], v[:, a], i[:, a], f[:, a]) for a in range(H)], dim=1)
    o = unit_rms(o, eps).reshape(T, H * e) * w[pre + "norm"] * torch.sigmoid(h @ w[pre + "g"].T)
    return o @ w[pre + "o"].T


def turn_half_split(v, base, dims):
    """v [T, ..., n]: column i pairs with column i + dims / 2 (i < dims / 2), the pair turned by the token's position
    times base^(-2i / dims); columns from dims on pass."""
    T = v.shape[0]
    i = torch.arange(dims // 2, dtype=v.dtype)
    a = torch.arange(T, dtype=v.dtype)[:, None] * base ** (-2.0 * i / max(dims, 1))[None, :]
    a = a.view([T] + [1] * (v.dim() - 2) + [dims // 2])
    c, s = torch.cos(a), torch.sin(a)
    half = dims // 2
    out = v.clone()
    x, y = v[..., :half], v[..., half:dims]
    out[..., :half] = x * c - y * s
    out[..., half:dims] = y * c + x * s
    return out


def causal_softmax(scores):
    T = scores.shape[0]
    see = torch.arange(T)[:, None] >= torch.arange(T)[None, :]
    return torch.softmax(scores.masked_fill(~see, -math.inf), dim=-1)


def latent_attention_mixer(h, w, pre, m, eps):
    T = h.shape[0]
    H, d, r, e, R = m["heads"], m["dim"], m["rot_dim"], m.get("vdim", m["dim"]), m["kv_rank"]
    q = (h @ w[pre + "q"].T).view(T, H, d + r)
    ckr = h @ w[pre + "dkv"].T
    c = unit_rms(ckr[:, :R], eps) * w[pre + "dkv.norm"]
    k_rot, q_rot = ckr[:, R:], q[..., d:]
    if r > 0:
        k_rot = turn_half_split(k_rot, m["rot"]["base"], m["rot"]["dims"])
        q_rot = turn_half_split(q_rot, m["rot"]["base"], m["rot"]["dims"])
    k = (c @ w[pre + "uk"].T).view(T, H, d)
    v = (c @ w[pre + "uv"].T).view(T, H, e)
    gate = torch.sigmoid(h @ w[pre + "g"].T)
    out = []
    for a in range(H):
        scores = (q[:, a, :d] @ k[:, a].T + q_rot[:, a] @ k_rot.T) * m["scale"]
        out.append(causal_softmax(scores) @ v[:, a] * gate[:, a:a + 1])
    return torch.cat(out, dim=1) @ w[pre + "o"].T


# -- feed-forwards -----------------------------------------------------------------------------------
def dense_ff(h, w, pre):
    return torch.relu(h @ w[pre + "up"].T) ** 2 @ w[pre + "down"].T


def gelu_exact(z):
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def expert(h, w, pre):
    return gelu_exact(h @ w[pre + "up"].T) @ w[pre + "down"].T


def router_scores(h, w, pre):
    return torch.softmax(h @ w[pre + "router"].T, dim=-1)


def chosen_experts(choice, top):
    """Per token the indices of the `top` largest choice scores (the lower index wins a tie)."""
    return [sorted(range(len(row)), key=lambda e: (-float(row[e]), e))[:top] for row in choice]


def routed_experts(h, w, pre, mlp):
    s = router_scores(h, w, pre)
    chosen = chosen_experts(s + w[pre + "correction"], mlp["router"]["top"])
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e in chosen[t]:
            own = e < mlp["router"]["experts"]
            y[t] += s[t, e] * (expert(h[t:t + 1], w, pre + "e%d." % e)[0] if own else h[t])
    return y


def feed_forward(h, w, pre, mlp):
    return dense_ff(h, w, pre) if mlp.get("kind", "dense") == "dense" else routed_experts(h, w, pre, mlp)


# -- the model ---------------------------------------------------------------------------------------
MIXERS = {"mlstm": mlstm_mixer, "latent_attention": latent_attention_mixer}


def mixed(x, w, i, lc, cfg, seen=lambda x: x):
    """The stream behind layer i's mixer. `seen`: what a sub-layer sees of the stream (the stream itself; a test may disturb
    it to learn how much a position's logits move)."""
    eps, L = cfg["norm"]["eps"], "l%d." % i
    return x + layer_norm(MIXERS[lc["type"]](seen(x), w, L + "mix.", lc["mixer"], eps), w[L + "norm1"], eps)


def layer(x, w, i, lc, cfg, seen=lambda x: x):
    x = mixed(x, w, i, lc, cfg, seen)
    if lc.get("mlp") is not None:
        x = x + layer_norm(feed_forward(seen(x), w, "l%d.mlp." % i, lc["mlp"]), w["l%d.norm2" % i], cfg["norm"]["eps"])
    return x


def streams(cfg, w, tokens: List[int], seen=lambda x: x):
    """The residual stream behind every layer, [layers, T, D]."""
    x = w["embed"][torch.tensor(tokens)]
    out = []
    for i, lc in enumerate(cfg["layers"]):
        x = layer(x, w, i, lc, cfg, seen)
        out.append(x)
    return torch.stack(out)


def logits(cfg, w, tokens: List[int], seen=lambda x: x):
    x = streams(cfg, w, tokens, seen)[-1]
    return layer_norm(x, w["final.norm"], cfg["norm"]["eps"]) @ w["head"].T * cfg.get("logit_scale", 1.0)


def closest_call(cfg, w, tokens: List[int], slight: float = 0.01):
    """Per token the smallest gap between the last chosen and the first rejected choice score over all routed layers
    (a tiny gap means rounding may choose another expert there); a call between two experts whose weights would both
    stay below `slight` does not count."""
    x = w["embed"][torch.tensor(tokens)]
    gap = torch.full((len(tokens),), math.inf, dtype=torch.float64)
    for i, lc in enumerate(cfg["layers"]):
        mlp = lc.get("mlp")
        if mlp is not None and mlp.get("kind") == "moe":
            r = mlp["router"]
            if r["top"] < r["experts"] + r.get("identity", 0):
                pre = "l%d.mlp." % i
                s = router_scores(mixed(x, w, i, lc, cfg), w, pre)
                srt = torch.sort(s + w[pre + "correction"], dim=-1, descending=True)
                at = slice(r["top"] - 1, r["top"] + 1)
                call = srt.values[:, r["top"] - 1] - srt.values[:, r["top"]]
                matters = torch.gather(s, 1, srt.indices[:, at]).max(dim=1).values >= slight
                gap = torch.where(matters, torch.minimum(gap, call), gap)
        x = layer(x, w, i, lc, cfg)
    return gap


def greedy_generate(cfg, w, prompt: List[int], n_new: int) -> List[int]:
    toks = list(prompt)
    for _ in range(n_new):
        toks.append(int(torch.argmax(logits(cfg, w, toks)[-1])))
    return toks[len(prompt):]
