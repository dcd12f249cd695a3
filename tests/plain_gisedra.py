"""A plain, slow Gisedra: whole sequences, no cache, one function for each mechanism.

Gisedra is a decoder-only model whose layers are listed in its configuration; a group of them may run several times with
the same weights, each run on a stream to which the embedding's output (from the second run on) and a vector of that
run are added. Every sub-layer stands between two dynamic tanh norms, ``x += n1b(mixer(n1(x))); x += n2b(ff(n2(x)))`` with
``n(x) = tanh(alpha x) w + b``, and behind them every layer adds an RMS-normed vector made from the stream and the
token's own row of a second table. A mixer is one of two:

* ``latent_attention``: keys and values of all heads expanded from one normed latent row per token, one rotated key part
  (interleaved pairs) that the heads share, a sliding window;
* ``parallel``: two mixers on one input, added with fixed scales: windowed softmax attention with grouped heads, a short
  causal convolution over queries, keys and values, a partial half-split rotation with scaled frequencies, kept first
  positions and a gate per output column; and retention (linear attention with one fixed decay per head).

The feed-forward is a mixture of gated experts (silu) whose weights are a softmax over the chosen router logits.
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
def dynamic_tanh(x, w, name):
    return torch.tanh(w[name + ".alpha"].reshape(()) * x) * w[name] + w[name + ".b"]


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z / (1.0 + torch.exp(-z))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def short_conv(u, taps):
    """u [T, C], taps [C, n]: channel by channel over time, the last tap the token's own, zeros in front."""
    T, n = u.shape[0], taps.shape[1]
    y = torch.zeros_like(u)
    for back in range(min(n, T)):
        y[back:] += taps[:, n - 1 - back] * u[:T - back]
    return y


def frequencies(rot):
    """The angle per position of every pair. With rot["scaling"]: long wavelengths are divided by `factor`, short ones
    kept, the ones between blended."""
    dims = rot["dims"]
    f = [rot["base"] ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if sc is None:
        return f
    out = []
    for one in f:
        turn = 2.0 * math.pi / one
        if turn < sc["original"] / sc["high"]:
            out.append(one)
        elif turn > sc["original"] / sc["low"]:
            out.append(one / sc["factor"])
        else:
            s = (sc["original"] / turn - sc["low"]) / (sc["high"] - sc["low"])
            out.append((1.0 - s) * one / sc["factor"] + s * one)
    return out


def turn(v, rot, interleaved):
    """v [T, ..., n]: pairs of the first rot["dims"] columns turned by the token's position times the pair's frequency;
    pairs (2i, 2i + 1), or (i, i + dims / 2)."""
    dims = rot["dims"]
    if dims == 0:
        return v
    T = v.shape[0]
    f = torch.tensor(frequencies(rot), dtype=v.dtype)
    a = (torch.arange(T, dtype=v.dtype)[:, None] * f[None, :]).view([T] + [1] * (v.dim() - 2) + [dims // 2])
    c, s = torch.cos(a), torch.sin(a)
    one = slice(0, dims, 2) if interleaved else slice(0, dims // 2)
    two = slice(1, dims, 2) if interleaved else slice(dims // 2, dims)
    out = v.clone()
    out[..., one] = v[..., one] * c - v[..., two] * s
    out[..., two] = v[..., two] * c + v[..., one] * s
    return out


def visible(T, mask):
    """[T, T]: whether position i sees position j."""
    back = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    see = back >= 0
    if mask is not None:
        see = see & ((back < mask["size"]) | (torch.arange(T)[None, :] < mask.get("keep_first", 0)))
    return see


def softmax_over(scores, see):
    return torch.softmax(scores.masked_fill(~see, -math.inf), dim=-1)


# -- mixers ------------------------------------------------------------------------------------------
def grouped_attention(h, w, pre, m):
    T = h.shape[0]
    H, d = m["heads"], m["dim"]
    G, e = m.get("kv_heads", H), m.get("vdim", d)
    p = {}
    for name in ("q", "k", "v"):
        p[name] = h @ w[pre + name].T
        if m.get("conv"):
            p[name] = short_conv(p[name], w[pre + name + ".conv"])
    q, k, v = p["q"].view(T, H, d), p["k"].view(T, G, d), p["v"].view(T, G, e)
    if m.get("rot") is not None:
        q, k = turn(q, m["rot"], False), turn(k, m["rot"], False)
    see = visible(T, m.get("mask"))
    out = [softmax_over(q[:, a] @ k[:, a // (H // G)].T * m["scale"], see) @ v[:, a // (H // G)] for a in range(H)]
    return (torch.cat(out, dim=1) * torch.sigmoid(h @ w[pre + "g"].T)) @ w[pre + "o"].T


def retention_readout(q, k, v, decay):
    """One head, token by token: q, k [T, d], v [T, e] -> [T, e]."""
    S = torch.zeros(q.shape[1], v.shape[1], dtype=q.dtype)
    out = torch.zeros(q.shape[0], v.shape[1], dtype=q.dtype)
    for t in range(q.shape[0]):
        S = decay * S + torch.outer(k[t], v[t])
        out[t] = S.T @ q[t]
    return out


def retention(h, w, pre, m, eps):
    T = h.shape[0]
    H, d = m["heads"], m["dim"]
    e = m.get("vdim", d)
    q = (h @ w[pre + "q"].T).view(T, H, d)
    k = (h @ w[pre + "k"].T).view(T, H, d) * d ** -0.5
    v = (h @ w[pre + "v"].T).view(T, H, e)
    o = torch.stack([retention_readout(q[:, a], k[:, a], v[:, a], m["decay"][a]) for a in range(H)], dim=1)
    return (unit_rms(o, eps).reshape(T, H * e) * silu(h @ w[pre + "g"].T)) @ w[pre + "o"].T


def parallel_mixer(h, w, pre, m, eps):
    return (m["left_scale"] * grouped_attention(h, w, pre + "left.", m["left"]) +
            m["right_scale"] * retention(h, w, pre + "right.", m["right"], eps))


def latent_attention(h, w, pre, m, eps):
    T = h.shape[0]
    H, d, r, R = m["heads"], m["dim"], m["rot_dim"], m["kv_rank"]
    e = m.get("vdim", d)
    q = (h @ w[pre + "q"].T).view(T, H, d + r)
    ckr = h @ w[pre + "dkv"].T
    c = unit_rms(ckr[:, :R], eps) * w[pre + "dkv.norm"]
    k_rot, q_rot = ckr[:, R:], q[..., d:]
    if r > 0:
        k_rot, q_rot = turn(k_rot, m["rot"], True), turn(q_rot, m["rot"], True)
    k = (c @ w[pre + "uk"].T).view(T, H, d)
    v = (c @ w[pre + "uv"].T).view(T, H, e)
    see = visible(T, m.get("mask"))
    out = [softmax_over((q[:, a, :d] @ k[:, a].T + q_rot[:, a] @ k_rot.T) * m["scale"], see) @ v[:, a] for a in range(H)]
    return torch.cat(out, dim=1) @ w[pre + "o"].T


def mixer(h, w, pre, lc, eps):
    return (parallel_mixer if lc["type"] == "parallel" else latent_attention)(h, w, pre, lc["mixer"], eps)


# -- feed-forward and the token's own input -----------------------------------------------------------
def router_logits(h, w, pre):
    return h @ w[pre + "router"].T + w[pre + "router.b"]


def chosen_experts(z, top):
    """Per token the indices of the `top` largest logits (the lower index wins a tie)."""
    return [sorted(range(len(row)), key=lambda e: (-float(row[e]), e))[:top] for row in z]


def expert(h, w, pre):
    return (silu(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def routed_experts(h, w, pre, mlp):
    z = router_logits(h, w, pre)
    y = torch.zeros_like(h)
    for t, chosen in enumerate(chosen_experts(z, mlp["router"]["top"])):
        weights = torch.softmax(z[t, chosen], dim=-1)
        for a, e in zip(weights, chosen):
            y[t] += a * expert(h[t:t + 1], w, pre + "e%d." % e)[0]
    return y


def token_side(x, w, i, tokens, dim, eps):
    L = "l%d.side." % i
    e = w["side.embed"][torch.tensor(tokens)][:, i * dim:(i + 1) * dim]
    y = (gelu_tanh(x @ w[L + "gate"].T) * e) @ w[L + "proj"].T
    return unit_rms(y, eps) * w[L + "norm"]


# -- the model ---------------------------------------------------------------------------------------
def order(cfg):
    """The layer runs as (layer, pass or None): a pass number stands at the first layer of each run of the loop."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if loop is None:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    runs = [(i, None) for i in range(a)]
    for t in range(loop["times"]):
        runs += [(i, t if i == a else None) for i in range(a, b)]
    return runs + [(i, None) for i in range(b, n)]


def mixed(x, w, i, lc, cfg, seen=lambda x: x):
    """The stream behind layer i's mixer. `seen`: what a sub-layer sees of the stream (the stream itself; a test may disturb
    it to learn how much a position's logits move)."""
    L = "l%d." % i
    y = mixer(dynamic_tanh(seen(x), w, L + "norm1"), w, L + "mix.", lc, cfg["norm"]["eps"])
    return x + dynamic_tanh(y, w, L + "norm1b")


def layer(x, w, i, lc, cfg, tokens, seen=lambda x: x):
    L = "l%d." % i
    x = mixed(x, w, i, lc, cfg, seen)
    if lc.get("mlp") is not None:
        y = routed_experts(dynamic_tanh(seen(x), w, L + "norm2"), w, L + "mlp.", lc["mlp"])
        x = x + dynamic_tanh(y, w, L + "norm2b")
    if cfg.get("token_side") is not None:
        x = x + token_side(seen(x), w, i, tokens, cfg["token_side"]["dim"], cfg["norm"]["eps"])
    return x


def before_pass(x, x0, w, t):
    return (x if t == 0 else x + x0) + w["loop.step"][t]


def streams(cfg, w, tokens: List[int], seen=lambda x: x):
    """The residual stream behind every layer run, [runs, T, D]."""
    x0 = w["embed"][torch.tensor(tokens)]
    x = x0
    out = []
    for i, t in order(cfg):
        if t is not None:
            x = before_pass(x, x0, w, t)
        x = layer(x, w, i, cfg["layers"][i], cfg, tokens, seen)
        out.append(x)
    return torch.stack(out)


def logits(cfg, w, tokens: List[int], seen=lambda x: x):
    return dynamic_tanh(streams(cfg, w, tokens, seen)[-1], w, "final.norm") @ w["head"].T


def closest_call(cfg, w, tokens: List[int]):
    """Per token the smallest gap between the last chosen and the first rejected router logit over all layer runs (a tiny
    gap means rounding may choose another expert there)."""
    x0 = w["embed"][torch.tensor(tokens)]
    x = x0
    gap = torch.full((len(tokens),), math.inf, dtype=torch.float64)
    for i, t in order(cfg):
        lc = cfg["layers"][i]
        if t is not None:
            x = before_pass(x, x0, w, t)
        mlp = lc.get("mlp")
        if mlp is not None and mlp["router"]["top"] < mlp["router"]["experts"]:
            h = dynamic_tanh(mixed(x, w, i, lc, cfg), w, "l%d.norm2" % i)
            z = torch.sort(router_logits(h, w, "l%d.mlp." % i), dim=-1, descending=True).values
            top = mlp["router"]["top"]
            gap = torch.minimum(gap, z[:, top - 1] - z[:, top])
        x = layer(x, w, i, lc, cfg, tokens)
    return gap


def greedy_generate(cfg, w, prompt: List[int], n_new: int) -> List[int]:
    toks = list(prompt)
    for _ in range(n_new):
        toks.append(int(torch.argmax(logits(cfg, w, toks)[-1])))
    return toks[len(prompt):]
